"""Vupolix through the step function, the cache and the model wiring on the CPU, with the GPU kernels replaced
by their plain torch stand-ins (tests/kernel_refs.py): packing, page tables and a ring that wraps, prompts longer
than the ring (whole and in portions), the states' slots (cleared when handed out, carried from step to step),
passes of repeated layers with lines of their own, which rows get logits; and the layers beside layers of other
arrangements."""
import copy

import pytest
import torch

import kernel_refs
import plain_vupolix as P
from vupolix_tiny import CONFIGS, MIXED, ODD, REPEATED, weights64, write_model
from tiny import random_ids

import inferllm_amd as I
from inferllm_amd.cache import CacheManager
from inferllm_amd.engine import DecoderModel, StepEntry, StepRunner
from inferllm_amd.weights.loader import stored_shapes


def build_runner(d, weights, max_tokens=1024, max_slots=3, max_seq_len=512, step_rows=0, change=None):
    cfg = I.load_config(d).with_tensor_shapes(stored_shapes(d))
    spec = cfg.to_spec()
    if change is not None:
        change(spec)
    model = DecoderModel(spec)
    model.load({k: v.to(torch.float32) for k, v in weights.items() if k in model.wants()})
    cache = CacheManager(model.kv_lines(), model.state_lines(), max_tokens=max_tokens, max_slots=max_slots,
                         max_seq_len=max_seq_len, dtype=torch.float32, device="cpu", poison_freed=True,
                         step_rows=step_rows)
    return StepRunner(model, cache, torch.float32, torch.device("cpu"), use_graphs=False)


@pytest.fixture
def emulated(monkeypatch):
    kernel_refs.patch(monkeypatch)


def near(got, want, tol=2e-4):
    assert float((got.double() - want).abs().max() / want.abs().max()) < tol


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompts_tokens_and_portions_equal_plain(name, tmp_path, emulated):
    config = CONFIGS[name]
    d = write_model(tmp_path, config, seed=2)
    w = weights64(d)
    r = build_runner(d, w)
    reqs = [random_ids(n, config["vocab"], 3 + n) for n in (170, 5, 21)]
    plain = [P.forward(config, w, ids) for ids in reqs]
    slots = [r.cache.alloc_slot() for _ in reqs]
    cut = [len(ids) - 3 for ids in reqs]
    out = r.step([StepEntry(s, ids[:k], [0, k - 1]) for s, ids, k in zip(slots, reqs, cut)])
    for i in range(3):
        near(out[2 * i:2 * i + 2], plain[i][[0, cut[i] - 1]])
    for t in range(3):
        live = [i for i in range(3) if not (i == 1 and t == 2)]
        if t == 2:
            r.cache.free_slot(slots[1])
        out = r.step([StepEntry(slots[i], [reqs[i][cut[i] + t]], [0]) for i in live])
        for j, i in enumerate(live):
            near(out[j], plain[i][cut[i] + t])
    for i in (0, 2):
        r.cache.free_slot(slots[i])
    # a prompt in portions of one, two and more tokens (across a window's and a page's border, past the
    # ring's end), in a slot, states and pages that were used before
    s = r.cache.alloc_slot()
    at, rows = 0, []
    for c in (1, 3, 5, 6, 30, 37, 39, 64, 66, 72, 127, 129, 170):
        rows.append(r.step([StepEntry(s, reqs[0][at:c], list(range(c - at)))]))
        at = c
    near(torch.cat(rows), plain[0])
    r.cache.free_slot(s)
    r.cache.check()


def test_the_ring_is_active_in_these_tests(tmp_path, emulated):
    d = write_model(tmp_path, ODD, seed=3)
    r = build_runner(d, weights64(d))
    assert sorted(g.ring for g in r.cache.groups) == [2, 2] and sum(len(g.lines) for g in r.cache.groups) == 6


def test_a_pass_keeps_what_is_its_own(tmp_path, emulated):
    """Another number of passes, other layers in them and no passes at all give what the plain model
    gives, and each something else: no pass reads another one's cache."""
    seen = []
    for loop in (None, (0, 4, 2), (1, 2, 3), (3, 4, 2)):
        config = copy.deepcopy(MIXED)
        config.pop("loop")
        if loop:
            config["loop"] = dict(zip(("start", "stop", "times"), loop))
        d = write_model(tmp_path, config, seed=8)
        w = weights64(d)
        r = build_runner(d, w)
        ids = random_ids(20, config["vocab"], 9)
        s = r.cache.alloc_slot()
        out = torch.cat([r.step([StepEntry(s, ids[:17], list(range(17)))])]
                        + [r.step([StepEntry(s, [t], [0])]) for t in ids[17:]])
        near(out, P.forward(config, w, ids))
        assert all(float((out - o).abs().max()) > 1e-2 for o in seen)
        seen.append(out)


def test_beside_layers_of_another_arrangement(tmp_path, emulated):
    """A plain pre-norm layer in the stretch that runs twice: the embedding is added to whatever the layer before
    left, pieces or a tensor, and the pieces are formed by whatever norm comes next."""
    from inferllm_amd.config.spec import PartSpec
    config = copy.deepcopy(REPEATED)
    config["layers"] = [config["layers"][0], copy.deepcopy(config["layers"][0])]
    config["loop"] = {"start": 0, "stop": 2, "times": 2}
    d = write_model(tmp_path, config, seed=4)
    w = weights64(d)
    E, eps, gain = config["width"], config["norm"]["eps"], config["residual_mult"]

    def change(spec):
        one = spec.layers[1]
        one.block, one.block_params, one.block_tensors = "pre_norm", {}, {}
        one.feed_forward = PartSpec("dense_activation", {"hidden_size": E, "intermediate_size": 64},
                                    {"up": "l1.mlp.e0.up", "down": "l1.mlp.e0.down"})
    r = build_runner(d, w, change=change)
    ids = random_ids(14, config["vocab"], 5)
    norm = lambda x, n: P.unit_rms(x, eps) * w[n]
    first = norm(w["embed"][torch.tensor(ids)], "embed.norm")
    x, m = first, config["layers"][0]["mixer"]
    for turn in range(2):
        x = x + first if turn else x
        x = x + gain * norm(P.wkv(norm(x, "l0.norm1"), w, "l0.mix.", m, eps), "l0.norm1b")
        x = x + gain * norm(P.experts(norm(x, "l0.norm2"), w, "l0.mlp.", config["layers"][0]["mlp"]), "l0.norm2b")
        x = x + P.wkv(norm(x, "l1.norm1"), w, "l1.mix.", m, eps)
        x = x + torch.clamp(norm(x, "l1.norm2") @ w["l1.mlp.e0.up"].T, min=0) ** 2 @ w["l1.mlp.e0.down"].T
    want = norm(x, "final.norm") @ w["head"].T * config["logit_scale"]
    out = r.step([StepEntry(r.cache.alloc_slot(), ids, list(range(14)))])
    near(out, want)
