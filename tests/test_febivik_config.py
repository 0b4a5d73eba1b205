"""Febivik's configuration: keys, checks, the translation into parts, sizes taken from a folder's
tensors, and the round trip through config.json."""
import copy

import pytest
import torch

import inferllm_amd as I
from inferllm_amd.config.registry import ConfigError
from inferllm_amd.engine import DecoderModel
from inferllm_amd.parts.position import scaled_frequencies
from febivik_tiny import CONFIGS, MIXED, ODD


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_round_trip_and_spec(name):
    cfg = I.config_from_dict(CONFIGS[name])
    assert type(cfg).__name__ == "FebivikConfig"
    assert I.config_from_dict(cfg.to_dict()).to_dict() == cfg.to_dict()
    spec = cfg.to_spec()
    assert len(spec.layers) == len(CONFIGS[name]["layers"])
    assert all(l.block == "post_norm" and l.mixer_norm.kind == "layer_norm" for l in spec.layers)
    DecoderModel(spec)


def test_tensors_by_kind_of_layer():
    wants = DecoderModel(I.config_from_dict(MIXED).to_spec()).wants()
    assert wants["l0.mix.q.norm"].shape == (20,) and wants["l0.mix.v.b"].shape == (2 * 12,)
    assert wants["l0.mlp.e4.down"].shape == (96, 56) and "l0.mlp.e0.gate" not in wants
    assert wants["l0.mlp.shared.up"].shape == (72, 96) and "l2.mlp.shared.up" not in wants
    assert wants["l1.mlp.act"].shape == (2,) and wants["l1.mix.norm"].shape == (3 * 28,)
    assert wants["l2.mix.w2"].shape == (2 * 24, 5) and wants["l2.mix.a.b"].shape == (48,)
    assert "l3.norm1.b" in wants and "l3.norm2" not in wants             # no feed-forward there
    assert wants["head"].shape == (310, 96)


def test_cache_needs():
    model = DecoderModel(I.config_from_dict(ODD).to_spec())
    kv = model.kv_lines()
    assert sorted(kv) == [1, 3] and sorted(model.state_lines()) == [0, 2]
    assert (kv[1].kind, kv[1].window, kv[1].keep_first) == ("window", 64, 1)
    assert (kv[3].window, kv[3].keep_first) == (29, 70)
    full = DecoderModel(I.config_from_dict(MIXED).to_spec()).kv_lines()[3]
    assert full.kind == "full" and full.window is None


def test_rank_comes_from_the_folders_tensors():
    d = copy.deepcopy(MIXED)
    del d["layers"][2]["mixer"]["rank"]
    cfg = I.config_from_dict(d).with_tensor_shapes({"l2.mix.w1": (11, 96)})
    assert cfg.layers[2]["mixer"]["rank"] == 11
    assert DecoderModel(cfg.to_spec()).wants()["l2.mix.w2"].shape == (48, 11)


def test_linear_scaling_divides_every_frequency():
    f, gain = scaled_frequencies(5000.0, 8, None)
    scaled, g2 = scaled_frequencies(5000.0, 8, {"factor": 3.0})
    assert gain == g2 == 1.0 and torch.allclose(scaled * 3.0, f, rtol=1e-15)


@pytest.mark.parametrize("edit, message", [
    (lambda d: d["layers"][0]["mixer"].update(kv_heads=4), "multiple of kv_heads"),
    (lambda d: d["layers"][0]["mixer"]["rot"].update(dims=22), "even and at most"),
    (lambda d: d["layers"][0]["mixer"]["mask"].update(keep_first=-1), "non-negative"),
    (lambda d: d["layers"][0]["mixer"]["rot"]["scaling"].update(factor=0), "positive"),
    (lambda d: d["layers"][1]["mixer"].update(decay=[0.5, 0.9]), "one number"),
    (lambda d: d["layers"][1]["mixer"].update(decay=[0.5, 0.9, 1.1]), "one number"),
    (lambda d: d["layers"][2]["mixer"].pop("dim"), "lacks"),
    (lambda d: d["layers"][2]["mlp"]["router"].update(top=7), "cannot be chosen"),
    (lambda d: d["layers"][1]["mlp"].update(kind="gated"), "not a feed-forward"),
    (lambda d: d["layers"][3].update(type="rnn"), "not a mixer"),
    (lambda d: d.pop("norm"), "lacks"),
])
def test_bad_configurations_are_refused(edit, message):
    d = copy.deepcopy(MIXED)
    edit(d)
    with pytest.raises(ConfigError, match=message):
        I.config_from_dict(d)
