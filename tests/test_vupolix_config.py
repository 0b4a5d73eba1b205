"""Vupolix's configuration: keys, checks, the translation into parts, the order in which repeated layers run,
sizes taken from a folder's tensors, and the round trip through config.json."""
import copy

import pytest
import torch

import inferllm_amd as I
from inferllm_amd.config.registry import ConfigError
from inferllm_amd.engine import DecoderModel
from vupolix_tiny import CONFIGS, MIXED, ODD, REPEATED


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_round_trip_and_spec(name):
    cfg = I.config_from_dict(CONFIGS[name])
    assert type(cfg).__name__ == "VupolixConfig"
    assert I.config_from_dict(cfg.to_dict()).to_dict() == cfg.to_dict()
    spec = cfg.to_spec()
    assert len(spec.layers) == len(CONFIGS[name]["layers"])
    assert all(l.block == "sandwich" and l.block_params["gain"] == CONFIGS[name]["residual_mult"] for l in spec.layers)
    assert spec.final_norm.params["scale"] == CONFIGS[name]["logit_scale"]
    DecoderModel(spec)


def runs(config):
    return [(e.layer, e.adds_embedding) for e in I.config_from_dict(config).to_spec().schedule]


def test_order_of_repeated_layers():
    assert runs(MIXED) == [(0, False), (1, False), (2, False), (1, True), (2, False), (3, False)]
    assert runs(ODD) == [(0, False), (1, False), (2, False), (0, True), (1, False), (2, False), (0, True), (1, False), (2, False)]
    assert runs(REPEATED) == [(0, False), (1, False), (2, False), (2, True)]
    once = copy.deepcopy(MIXED)
    once["loop"]["times"] = 1
    none = copy.deepcopy(MIXED)
    del none["loop"]
    assert runs(once) == runs(none) == [(i, False) for i in range(4)]


def test_every_run_has_a_cache_and_a_state_of_its_own():
    model = DecoderModel(I.config_from_dict(MIXED).to_spec())
    kv, states = model.kv_lines(), model.state_lines()
    assert sorted(kv) == [0, 2, 4] and sorted(states) == [0, 1, 2, 3, 4, 5]
    assert (kv[0].kind, kv[0].window) == ("window", 37) and kv[2] == kv[4] and kv[2].kind == "full"
    assert states[1]["S"].shape == (3, 24, 24) and states[1]["tail"].shape == (1, 96) and states[3] == states[1]
    assert set(states[0]) == {"S"} and states[0]["S"].shape == (3, 16, 28)


def test_tensors_by_kind_of_layer():
    wants = DecoderModel(I.config_from_dict(MIXED).to_spec()).wants()
    assert wants["l0.mix.left.k"].shape == (2 * 20, 96) and "l0.mix.left.v" not in wants
    assert wants["l0.mix.left.g"].shape == (6, 96) and wants["l0.mix.left.sink"].shape == (6,)
    assert wants["l0.mix.right.g"].shape == (3 * 28, 96) and wants["l0.mix.right.out"].shape == (96,)
    assert wants["l1.mix.mu.g"].shape == (96,) and wants["l1.mix.u"].shape == (3, 24) and wants["l1.mix.w2"].shape == (72, 5)
    assert wants["l0.mlp.e7.up"].shape == (56, 96) and wants["l0.mlp.correction"].shape == (8,)
    assert wants["l0.mlp.shared.down"].shape == (96, 72) and "l1.mlp.shared.up" not in wants
    assert "l2.norm1b" in wants and "l2.norm2" not in wants              # no feed-forward there
    assert wants["embed.norm"].shape == (96,) and wants["head"].shape == (310, 96)


def test_what_a_folders_tensors_state():
    d = copy.deepcopy(MIXED)
    del d["layers"][1]["mixer"]["rank"]
    cfg = I.config_from_dict(d).with_tensor_shapes({"l1.mix.w1": (11, 96), "l2.norm2": (96,), "l2.norm2b": (96,)})
    assert cfg.layers[1]["mixer"]["rank"] == 11
    assert DecoderModel(cfg.to_spec()).wants()["l1.mix.w2"].shape == (72, 11)
    assert cfg.to_spec().ignored_tensor_suffixes == ["l2.norm2", "l2.norm2b"]


def test_a_run_that_adds_the_embedding_again_adds_to_whatever_is_left():
    """`ops.plus_rows` over everything a block may leave to be added."""
    import kernel_refs
    from inferllm_amd.kernels import ops
    mp = pytest.MonkeyPatch()
    kernel_refs.patch(mp)
    try:
        g = torch.Generator().manual_seed(1)
        e, a, b, w = (torch.randn(3, 8, generator=g) for _ in range(4))
        w = w[0]
        assert ops.plus_rows(None, e) is e
        assert torch.equal(ops.plus_rows(a, e), a + e)
        assert torch.equal(ops.plus_rows((a, b), e), (a + b) + e)
        left = ops.PostNormed(a, w, 1e-5, 0.7)
        both = ops.plus_rows(ops.plus_rows(left, e), b)
        want = left.tensor() + e + b
        assert not both.plain and torch.allclose(both.tensor(), want, atol=1e-6)
        x = torch.randn(3, 8, generator=g)
        moved = x.clone()
        ops.post_add_norm(moved, both, None, None, None, 0.0, None)
        assert torch.allclose(moved, x + want, atol=1e-6)
        with pytest.raises(ops.KernelError, match="cannot be added"):
            ops.plus_rows(object(), e)
    finally:
        mp.undo()


@pytest.mark.parametrize("edit, message", [
    (lambda d: d["layers"][0]["mixer"]["left"].update(kv_heads=4), "multiple of kv_heads"),
    (lambda d: d["layers"][0]["mixer"]["left"].update(vdim=24), "must equal dim"),
    (lambda d: d["layers"][0]["mixer"]["left"]["rot"].update(dims=22), "even and at most"),
    (lambda d: d["layers"][0]["mixer"]["left"]["rot"]["scaling"].pop("fast"), "lacks"),
    (lambda d: d["layers"][0]["mixer"]["left"]["mask"].update(size=0), "positive integer"),
    (lambda d: d["layers"][0]["mixer"]["right"].update(decay=[0.5, 0.9]), "one number"),
    (lambda d: d["layers"][0]["mixer"]["right"].update(decay=[0.5, 0.9, 1.1]), "one number"),
    (lambda d: d["layers"][1]["mixer"].pop("dim"), "lacks"),
    (lambda d: d["layers"][0]["mlp"]["router"].update(top=5), "cannot be chosen"),
    (lambda d: d["layers"][0]["mlp"]["router"]["groups"].update(count=3), "equal groups"),
    (lambda d: d["layers"][0]["mlp"]["router"]["groups"].update(keep=5), "equal groups"),
    (lambda d: d["layers"][1]["mlp"].update(kind="dense"), "not a feed-forward"),
    (lambda d: d["layers"][3].update(type="rnn"), "not a mixer"),
    (lambda d: d["loop"].update(stop=5), "cannot be repeated"),
    (lambda d: d["loop"].update(start=3), "cannot be repeated"),
    (lambda d: d["loop"].update(times=0), "positive integer"),
    (lambda d: d.pop("residual_mult"), "lacks"),
])
def test_bad_configurations_are_refused(edit, message):
    d = copy.deepcopy(MIXED)
    edit(d)
    with pytest.raises(ConfigError, match=message):
        I.config_from_dict(d)
