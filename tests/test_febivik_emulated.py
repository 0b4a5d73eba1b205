"""Febivik through the step function, the cache and the model wiring on the CPU, with the GPU kernels
replaced by their plain torch stand-ins (tests/kernel_refs.py): packing, page tables with kept first
pages and a ring that wraps, prompts longer than the ring (whole and in portions), the states' slots
(cleared when handed out, carried from step to step), which rows get logits; and blocks of different
arrangements one behind the other."""
import copy

import pytest
import torch

import kernel_refs
import plain_febivik as P
from febivik_tiny import CONFIGS, MIXED, ODD, weights64, write_model
from tiny import random_ids

import inferllm_amd as I
from inferllm_amd.cache import CacheManager
from inferllm_amd.cache.manager import KVGroup, KVSpec, TokenTensor
from inferllm_amd.cache.slots import CacheError
from inferllm_amd.engine import DecoderModel, StepEntry, StepRunner
from inferllm_amd.weights.loader import stored_shapes


def build_runner(d, weights, max_tokens=1024, max_slots=3, max_seq_len=512, step_rows=0):
    cfg = I.load_config(d).with_tensor_shapes(stored_shapes(d))
    model = DecoderModel(cfg.to_spec())
    model.load({k: v.to(torch.float32) for k, v in weights.items() if k in model.wants()})
    cache = CacheManager(model.kv_lines(), model.state_lines(), max_tokens=max_tokens, max_slots=max_slots,
                         max_seq_len=max_seq_len, dtype=torch.float32, device="cpu", poison_freed=True,
                         step_rows=step_rows)
    return StepRunner(model, cache, torch.float32, torch.device("cpu"), use_graphs=False)


@pytest.fixture
def emulated(monkeypatch):
    kernel_refs.patch(monkeypatch)


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompts_tokens_and_portions_equal_plain(name, tmp_path, emulated):
    config = CONFIGS[name]
    d = write_model(tmp_path, config, seed=2)
    w = weights64(d)
    r = build_runner(d, w)
    reqs = [random_ids(n, config["vocab"], 3 + n) for n in (290, 5, 21)]
    plain = [P.forward(config, w, ids) for ids in reqs]
    slots = [r.cache.alloc_slot() for _ in reqs]
    cut = [len(ids) - 3 for ids in reqs]
    out = r.step([StepEntry(s, ids[:k], [0, k - 1]) for s, ids, k in zip(slots, reqs, cut)])
    for i in range(3):
        assert (out[2 * i:2 * i + 2].double() - plain[i][[0, cut[i] - 1]]).abs().max() < 2e-4
    for t in range(3):
        live = [i for i in range(3) if not (i == 1 and t == 2)]
        if t == 2:
            r.cache.free_slot(slots[1])
        out = r.step([StepEntry(slots[i], [reqs[i][cut[i] + t]], [0]) for i in live])
        for j, i in enumerate(live):
            assert (out[j].double() - plain[i][cut[i] + t]).abs().max() < 2e-4
    for i in (0, 2):
        r.cache.free_slot(slots[i])
    # a prompt in portions of one, two and more tokens (across a window's and a page's border, past
    # the ring's end), in a slot, states and pages that were used before
    s = r.cache.alloc_slot()
    at, rows = 0, []
    for c in (1, 3, 5, 6, 30, 37, 39, 64, 66, 72, 127, 129, 200, 290):
        rows.append(r.step([StepEntry(s, reqs[0][at:c], list(range(c - at)))]))
        at = c
    assert (torch.cat(rows).double() - plain[0]).abs().max() < 2e-4
    r.cache.free_slot(s)
    r.cache.check()


def test_portions_as_long_as_the_ring_allows(tmp_path, emulated):
    """A portion of just the step function's limit stores every one of its rows, also those whose page
    of the ring the portion's last rows come close to."""
    d = write_model(tmp_path, ODD, seed=6)
    w = weights64(d)
    r = build_runner(d, w, step_rows=32)
    limit = r.cache.step_limit
    ids = random_ids(190 + 2 * limit, ODD["vocab"], 7)
    s = r.cache.alloc_slot()
    r.step([StepEntry(s, ids[:190], [])])
    got = r.step([StepEntry(s, ids[190:], list(range(2 * limit)))])      # (runs as two pieces)
    assert (got.double() - P.forward(ODD, w, ids)[190:]).abs().max() < 2e-4


def test_kept_pages_stay_ahead_of_the_ring():
    spec = KVSpec("window", (TokenTensor("k", (1, 4)),), 29, 70)
    g = KVGroup(spec, [0], n_slots=2, max_tokens=4096, max_seq_len=1024, dtype=torch.float32, device="cpu")
    assert (g.kept_pages, g.ring, g.pages_per_seq) == (2, 2, 4)
    assert g.step_limit == 2 * 64 - 29 + 1
    assert [g.pages_needed(n) for n in (1, 64, 65, 200, 1000)] == [1, 1, 2, 4, 4]
    g.reserve(0, 700)
    assert len(g.held[0]) == 4
    # a window that never wraps within the longest sequence keeps everything
    g = KVGroup(spec, [0], n_slots=2, max_tokens=4096, max_seq_len=256, dtype=torch.float32, device="cpu")
    assert (g.kept_pages, g.ring) == (0, 0) and g.step_limit is None
    with pytest.raises(CacheError, match="window"):
        KVSpec("full", (TokenTensor("k", (1, 4)),), None, 3)


def test_the_ring_is_active_in_these_tests(tmp_path, emulated):
    d = write_model(tmp_path, ODD, seed=3)
    r = build_runner(d, weights64(d))
    assert [(g.kept_pages, g.ring) for g in r.cache.groups] == [(1, 2), (2, 2)]


def test_post_norm_layers_beside_layers_with_norms_in_front(tmp_path, emulated):
    """The pieces that a layer with norms behind leaves are formed by whatever norm comes next: a
    pre-norm layer in the middle of the model and a last RMS norm give what the plain sums give."""
    from inferllm_amd.config.spec import PartSpec
    config = copy.deepcopy(MIXED)
    config["layers"] = [config["layers"][1], config["layers"][1], config["layers"][1]]
    d = write_model(tmp_path, config, seed=4)
    w = weights64(d)
    spec = I.load_config(d).to_spec()
    E, eps = config["width"], config["norm"]["eps"]
    rms = lambda n: PartSpec("rms_norm", {"size": E, "eps": eps}, {"weight": n})
    spec.layers[1].block, spec.layers[1].mixer_norm, spec.layers[1].feed_forward_norm = "pre_norm", rms("l1.norm1"), rms("l1.norm2")
    spec.final_norm = rms("final.norm")
    model = DecoderModel(spec)
    model.load({k: v.to(torch.float32) for k, v in w.items() if k in model.wants()})
    cache = CacheManager(model.kv_lines(), model.state_lines(), max_tokens=256, max_slots=1, max_seq_len=128,
                         dtype=torch.float32, device="cpu")
    r = StepRunner(model, cache, torch.float32, torch.device("cpu"), use_graphs=False)
    ids = random_ids(12, config["vocab"], 5)
    norm = lambda x, n: P.unit_rms(x, eps) * w[n]
    x = w["embed"][torch.tensor(ids)]
    for i, m in ((0, config["layers"][0]["mixer"]), (1, config["layers"][0]["mixer"]), (2, config["layers"][0]["mixer"])):
        p = f"l{i}."
        if i == 1:
            x = x + P.lightning(norm(x, p + "norm1"), w, p + "mix.", m, eps)
            x = x + P.dense(norm(x, p + "norm2"), w, p + "mlp.")
        else:
            x = x + P.layer_norm(P.lightning(x, w, p + "mix.", m, eps), w[p + "norm1"], w[p + "norm1.b"], eps)
            x = x + P.layer_norm(P.dense(x, w, p + "mlp."), w[p + "norm2"], w[p + "norm2.b"], eps)
    want = norm(x, "final.norm") @ w["head"].T
    out = r.step([StepEntry(cache.alloc_slot(), ids, list(range(12)))])
    assert (out.double() - want).abs().max() < 2e-4
