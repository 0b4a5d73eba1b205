"""Febivik through the engine against the plain model (tests/plain_febivik.py): every mechanism in
a layer of its own, whole prompts, token-by-token decoding, prompts cut into portions down to two
tokens, batches of unequal requests, slots, pages and states used again, planted keys far away, at
page borders, just inside and just outside a window and among the first tokens that a window keeps
(and the next one), in prompts and in decoding and past the end of the cache's ring, a memory from
far back, long decoding, greedy generation through the engine's own loop, the command line and the
trace replay; and the new kernels alone.  Configurations: tests/febivik_tiny.py."""
import json
import os

import pytest
import torch

import kernel_refs as R
import plain_febivik as P
from febivik_tiny import (CONFIGS, MIXED, NO_KEYS, ODD, _att, _delta, _dense, _light, _moe, _rot, plant_key,
                          plant_memory, single, weights64, write_model)
from tiny import random_ids

pytestmark = pytest.mark.gpu

BUDGET = {"float32": 3e-5, "bfloat16": 4e-2}
STORE = {"float32": torch.float32, "bfloat16": torch.bfloat16}


def engine_for(d, dtype, **kw):
    import inferllm_amd as I
    kw.setdefault("max_batch", 8)
    kw.setdefault("max_seq_len", 1024)
    kw.setdefault("poison_freed", True)
    return I.Engine.from_pretrained(d, dtype=dtype, device="cuda:0", **kw)


def feed(eng, slot, tokens, cuts):
    """Logits of every position of `tokens`, fed in steps that end at `cuts` (then one by one)."""
    from inferllm_amd import StepEntry
    rows, at = [], 0
    for c in list(cuts) + list(range((cuts[-1] if cuts else 0) + 1, len(tokens) + 1)):
        if c <= at:
            continue
        rows.append(eng.step([StepEntry(slot, tokens[at:c], list(range(c - at)))]).clone())
        at = c
    return torch.cat(rows)


def close(got, want, dtype, what=""):
    """float32: every row within the budget.  bfloat16: rounding of the activations can turn a
    router's close call, which moves one token's output (and through the states a little of the next
    ones'): all rows but a few within the budget, and the median well inside it."""
    scale = want.abs().max()
    err = (got.double().cpu() - want).abs().amax(dim=-1) / scale
    assert not torch.isnan(got).any(), what
    if dtype == "float32":
        assert float(err.max()) < BUDGET[dtype], (what, float(err.max()))
    else:
        over = int((err > BUDGET[dtype]).sum())
        assert over <= max(1, len(err) // 10) and float(err.median()) < BUDGET[dtype] / 2, \
            (what, over, len(err), float(err.median()))


# ------------------------------------------------------------------ each mechanism in a layer of its own
MECHANISMS = {
    "attention_part_rotated_grouped": single("attention", _att(6, 3, 16, 40, 0.3, _rot(700.0, 6, 2.5))),
    "attention_all_rotated_one_kv_head": single("attention", _att(5, 1, 24, 8, 0.4, _rot(20000.0, 24))),
    "attention_without_rotation": single("attention", _att(4, 2, 12, 20, 0.4)),
    "attention_wide_heads": single("attention", _att(2, 2, 136, 132, 0.1, _rot(100.0, 64, 4.0), 33, 5)),
    "window_alone": single("attention", _att(4, 2, 16, 16, 0.5, _rot(90.0, 8), 29)),
    "window_and_first_tokens": single("attention", _att(6, 2, 20, 12, 0.5, _rot(50.0, 10, 1.3), 23, 4)),
    "window_of_one": single("attention", _att(2, 1, 8, 24, 0.9, _rot(9.0, 8), 1, 2)),
    "lightning_wide_keys": single("lightning", _light(3, 40, 12, (0.9, 0.5, 0.99))),
    "lightning_wide_values": single("lightning", _light(2, 8, 72, (0.97, 0.3))),
    "lightning_sizes_of_two": single("lightning", _light(2, 10, 14, (1.0, 0.0))),
    "lightning_beyond_the_chunks": single("lightning", _light(2, 132, 136, (0.9, 0.99))),
    "delta_small": single("general_delta", _delta(3, 10, 2)),
    "delta_wide": single("general_delta", _delta(2, 132, 6)),
    "dense_feed_forward": single("lightning", _light(2, 8, 8, (0.9, 0.7)), _dense(88)),
    "experts_one_chosen": single("lightning", _light(2, 8, 8, (0.9, 0.7)), _moe(32, 5, 1, 3.0)),
    "experts_and_shared": single("lightning", _light(2, 8, 8, (0.9, 0.7)), _moe(40, 6, 3, 0.7, 52)),
    "experts_on_the_matrix_cores": single("lightning", _light(2, 8, 8, (0.9, 0.7)), _moe(64, 4, 2, 1.4, 96)),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(MECHANISMS))
def test_mechanism_alone_prompt_and_tokens(tmp_path_factory, name, dtype):
    """A one-layer model that has the mechanism: a prompt of 70 tokens, then 10 single tokens."""
    config = MECHANISMS[name]
    d = write_model(tmp_path_factory.getbasetemp(), config, seed=5, dtype=STORE[dtype])
    eng = engine_for(d, dtype)
    ids = random_ids(80, config["vocab"], 17)
    slot = eng.alloc_slot()
    close(feed(eng, slot, ids, [70]), P.forward(config, weights64(d), ids), dtype, name)
    eng.free_slot(slot)
    eng.cache.check()


# ------------------------------------------------------------------ whole models
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_prompts_of_unequal_lengths_then_tokens(tmp_path_factory, name, dtype):
    """Several prompts in one step (1 to 140 tokens, the first tokens of each included), then
    four steps of one token each for all of them, against the plain model of each alone."""
    from inferllm_amd import StepEntry
    config = CONFIGS[name]
    d = write_model(tmp_path_factory.getbasetemp(), config, seed=3, dtype=STORE[dtype])
    w = weights64(d)
    eng = engine_for(d, dtype)
    reqs = [random_ids(n + 4, config["vocab"], 11 * n) for n in (1, 2, 140, 65, 33, 71)]
    slots = [eng.alloc_slot() for _ in reqs]
    got = [[] for _ in reqs]
    out = eng.step([StepEntry(s, r[:-4], list(range(len(r) - 4))) for s, r in zip(slots, reqs)])
    at = 0
    for i, r in enumerate(reqs):
        got[i].append(out[at:at + len(r) - 4].clone())
        at += len(r) - 4
    for t in (4, 3, 2, 1):
        out = eng.step([StepEntry(s, [r[-t]], [0]) for s, r in zip(slots, reqs)])
        for i in range(len(reqs)):
            got[i].append(out[i:i + 1].clone())
    for i, r in enumerate(reqs):
        close(torch.cat(got[i]), P.forward(config, w, r), dtype, f"request {i}")
    for s in slots:
        eng.free_slot(s)
    eng.cache.check()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cuts", [[], [1], [2, 4, 6], [36, 37, 38, 63, 64, 65, 130], [17, 19, 100], [128], [140]])
def test_token_by_token_and_portions_equal_the_whole_prompt(tmp_path_factory, cuts, dtype):
    """140 tokens one by one ([]), or in portions that end at `cuts` (portions of one and two
    tokens, portions that end at, before and after a window's, a chunk's and a page's border) and
    then one by one."""
    d = write_model(tmp_path_factory.getbasetemp(), MIXED, seed=4, dtype=STORE[dtype])
    eng = engine_for(d, dtype)
    ids = random_ids(140, MIXED["vocab"], 23)
    want = P.forward(MIXED, weights64(d), ids)
    slot = eng.alloc_slot()
    close(feed(eng, slot, ids if cuts else ids[:45], cuts), want if cuts else want[:45], dtype, str(cuts))
    eng.free_slot(slot)
    eng.cache.check()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cuts", [[500], [150, 152, 290, 500], [60, 61, 320], [1, 200]])
def test_prompts_longer_than_the_ring(tmp_path_factory, cuts, dtype):
    """500 tokens and more through a ring of a few pages: whole, in portions (cut further by the step
    function where they would write round the ring) and token by token, kept pages in front."""
    d = write_model(tmp_path_factory.getbasetemp(), ODD, seed=19, dtype=STORE[dtype])
    eng = engine_for(d, dtype, step_rows=32)
    assert all(g.ring and g.kept_pages for g in eng.cache.groups)
    n = 510 if cuts[-1] == 500 else cuts[-1] + 20
    ids = random_ids(n, ODD["vocab"], 29)
    want = P.forward(ODD, weights64(d), ids)
    slot = eng.alloc_slot()
    close(feed(eng, slot, ids, cuts), want, dtype, str(cuts))
    eng.free_slot(slot)
    eng.cache.check()


@pytest.mark.parametrize("dtype", ["float32"])
def test_mixed_steps_of_portions_starts_and_single_tokens(tmp_path_factory, dtype):
    """Steps that hold a sequence that starts, one that goes on by a portion and one that goes on
    by two tokens, against each alone; every mixer goes on from what it kept."""
    from inferllm_amd import StepEntry
    d = write_model(tmp_path_factory.getbasetemp(), ODD, seed=9, dtype=STORE[dtype])
    w = weights64(d)
    eng = engine_for(d, dtype)
    a, b, c = (random_ids(n, ODD["vocab"], n) for n in (90, 70, 30))
    sa, sb, sc = (eng.alloc_slot() for _ in range(3))
    rows = {"a": [], "b": [], "c": []}
    out = eng.step([StepEntry(sa, a[:50], list(range(50)))])
    rows["a"].append(out.clone())
    out = eng.step([StepEntry(sa, a[50:88], list(range(38))), StepEntry(sb, b[:66], list(range(66)))])
    rows["a"].append(out[:38].clone()); rows["b"].append(out[38:].clone())
    out = eng.step([StepEntry(sc, c, list(range(30))), StepEntry(sa, a[88:], [0, 1]),
                    StepEntry(sb, b[66:], list(range(4)))])
    rows["c"].append(out[:30].clone()); rows["a"].append(out[30:32].clone()); rows["b"].append(out[32:].clone())
    for name, ids in (("a", a), ("b", b), ("c", c)):
        close(torch.cat(rows[name]), P.forward(ODD, w, ids), dtype, name)
    for s in (sa, sb, sc):
        eng.free_slot(s)
    eng.cache.check()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_slots_and_pages_used_again(tmp_path_factory, dtype):
    """Requests come and go in a cache with little room: later ones run in slots, pages and states
    that earlier ones used (freed pages are poisoned), and equal what they give alone."""
    from inferllm_amd import StepEntry
    d = write_model(tmp_path_factory.getbasetemp(), MIXED, seed=6, dtype=STORE[dtype])
    w = weights64(d)
    eng = engine_for(d, dtype, max_batch=2, max_tokens=384, max_seq_len=256, step_rows=16)
    for round_ in range(3):
        reqs = [random_ids(n, MIXED["vocab"], 100 * round_ + n) for n in (100 + round_ * 30, 40 + round_)]
        slots = [eng.alloc_slot() for _ in reqs]
        out = eng.step([StepEntry(s, r[:-3], list(range(len(r) - 3))) for s, r in zip(slots, reqs)])
        got = [[out[:len(reqs[0]) - 3].clone()], [out[len(reqs[0]) - 3:].clone()]]
        for t in (3, 2, 1):
            out = eng.step([StepEntry(s, [r[-t]], [0]) for s, r in zip(slots, reqs)])
            got[0].append(out[:1].clone()); got[1].append(out[1:].clone())
        for i, r in enumerate(reqs):
            close(torch.cat(got[i]), P.forward(MIXED, w, r), dtype, f"pass {round_} request {i}")
        for s in slots:
            eng.free_slot(s)
        eng.cache.check()


@pytest.mark.parametrize("kind", ["lightning", "general_delta"])
def test_state_starts_at_zero_in_a_slot_used_before(tmp_path_factory, kind):
    """The state is cleared when a slot is handed out: the same request twice in the same slot gives
    the same bits, with another request between."""
    from inferllm_amd import StepEntry
    config = single(kind, _light(2, 16, 24, (0.99, 0.7)) if kind == "lightning" else _delta(3, 16, 4), _dense(32))
    d = write_model(tmp_path_factory.getbasetemp(), config, seed=2, dtype=torch.float32)
    eng = engine_for(d, "float32", max_batch=1)
    a, b = random_ids(80, config["vocab"], 1), random_ids(77, config["vocab"], 2)
    outs = []
    for ids in (a, b, a):
        slot = eng.alloc_slot()
        eng.step([StepEntry(slot, ids[:-1], [])])
        outs.append(eng.step([StepEntry(slot, ids[-1:], [0])]).clone())
        eng.free_slot(slot)
    assert torch.equal(outs[0], outs[2])
    close(outs[0], P.forward(config, weights64(d), a)[-1:], "float32")


def test_a_row_does_not_depend_on_its_batch(tmp_path_factory):
    """The same request decoded alone and among others of very different lengths: the same logits up
    to rounding."""
    from inferllm_amd import StepEntry
    d = write_model(tmp_path_factory.getbasetemp(), MIXED, seed=21, dtype=torch.float32)
    eng = engine_for(d, "float32")
    reqs = [random_ids(n, MIXED["vocab"], n) for n in (100, 3, 230, 41)]
    alone = []
    for r in reqs:
        s = eng.alloc_slot()
        eng.step([StepEntry(s, r[:-2], [])])
        alone.append(torch.cat([eng.step([StepEntry(s, [t], [0])]).clone() for t in r[-2:]]))
        eng.free_slot(s)
    slots = [eng.alloc_slot() for _ in reqs]
    eng.step([StepEntry(s, r[:-2], []) for s, r in zip(slots, reqs)])
    two = [eng.step([StepEntry(s, [r[t]], [0]) for s, r in zip(slots, reqs)]).clone() for t in (-2, -1)]
    for i in range(len(reqs)):
        close(torch.stack([two[0][i], two[1][i]]), alone[i].double().cpu(), "float32", f"request {i}")


# ------------------------------------------------------------------ far keys, window edges, kept first tokens
def _planted(tmp_path_factory, config, dtype, n, query_at, key_at, seed=8):
    KEY, QUERY = 250, 251
    ids = [t % 250 for t in random_ids(n, 250, 31)]
    ids[key_at] = KEY
    if query_at != key_at:
        ids[query_at] = QUERY
    edit = lambda w: plant_key(w, config, KEY, QUERY if query_at != key_at else KEY)
    d = write_model(tmp_path_factory.getbasetemp(), config, seed=seed, dtype=STORE[dtype], edit=edit)
    return d, ids


def _prompt_and_decoded(d, dtype, ids, want, query_at, **kw):
    eng = engine_for(d, dtype, **kw)
    slot = eng.alloc_slot()
    got = feed(eng, slot, ids, [len(ids)])
    close(got[[query_at]], want[[query_at]], dtype, "the query's row in a prompt")
    close(got, want, dtype, "prompt")
    eng.free_slot(slot)
    slot = eng.alloc_slot()
    got = feed(eng, slot, ids[:query_at + 3], [max(1, query_at - 2)])
    close(got[[query_at]], want[[query_at]], dtype, "the query's row decoded")
    close(got, want[:query_at + 3], dtype, "decoded")
    eng.free_slot(slot)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("query_at, key_at", [(399, 0), (399, 3), (300, 63), (300, 64), (257, 128), (1, 0), (5, 5)])
def test_a_planted_key_far_back_under_full_attention(tmp_path_factory, query_at, key_at, dtype):
    """One position's key is made to stand out for one query position hundreds of tokens later (at
    the sequence's first tokens, on both sides of page borders), in a prompt and as a decoded
    token; the same sequence without the key token gives logits far from the right ones."""
    config = single("attention", _att(4, 2, 16, 24, 1.0, _rot(10000.0, 8, 2.0)), _dense(40), vocab=260)
    d, ids = _planted(tmp_path_factory, config, dtype, 400, query_at, key_at)
    w = weights64(d)
    want = P.forward(config, w, ids)
    wrong = P.forward(config, w, ids[:key_at] + [7] + ids[key_at + 1:])
    moved = (wrong[query_at] - want[query_at]).abs().max() / want[query_at].abs().max()
    assert float(moved) > 8 * BUDGET[dtype], float(moved)
    _prompt_and_decoded(d, dtype, ids, want, query_at)


WINDOW, KEEP = 37, 5


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("step_rows", [16, 512])             # the ring wraps within the sequence, or never does
@pytest.mark.parametrize("query_at, key_at", [
    (110, 74), (110, 73),          # the window's last position, and the one beyond it
    (100, 64), (100, 63),          # the same on both sides of the page border at 64
    (293, 257), (293, 256), (164, 128), (164, 127),
    (110, 4), (110, 5), (293, 4), (293, 5), (293, 0),       # the last kept token, the first one not kept
    (41, 4), (41, 5), (42, 5), (37, 0), (5, 4), (1, 0),     # where the window has just left the kept tokens
])
def test_a_planted_key_at_the_edges_of_a_window_and_of_the_kept_tokens(tmp_path_factory, query_at, key_at, step_rows,
                                                                       dtype):
    """A key at the window's far edge is seen, one position further it is not; one of the first KEEP
    tokens is seen from anywhere, the next one is not.  A window, or a number of kept tokens, that is
    one off moves the logits by far more than the budget."""
    config = single("attention", _att(4, 2, 16, 24, 1.0, _rot(10000.0, 8, 2.0), WINDOW, KEEP), _dense(40), vocab=260)
    d, ids = _planted(tmp_path_factory, config, dtype, 300, query_at, key_at)
    w = weights64(d)
    want = P.forward(config, w, ids)
    dist = query_at - key_at
    if dist < WINDOW - 1 or (key_at < KEEP - 1):             # well inside: the sequence without the key token
        wrong = P.forward(config, w, ids[:key_at] + [7] + ids[key_at + 1:])
    elif key_at in (KEEP - 1, KEEP) and dist >= WINDOW:      # at the kept tokens' end
        wrong = P.forward(config, w, ids, keep_shift=-1 if key_at < KEEP else 1)
    else:                                                    # at the window's edge
        wrong = P.forward(config, w, ids, edge_shift=-1 if dist < WINDOW else 1)
    moved = (wrong[query_at] - want[query_at]).abs().max() / want[query_at].abs().max()
    assert float(moved) > 8 * BUDGET[dtype], float(moved)
    _prompt_and_decoded(d, dtype, ids, want, query_at, step_rows=step_rows)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["lightning", "general_delta"])
def test_a_memory_from_far_back(tmp_path_factory, kind, dtype):
    """A recurrent layer that hardly forgets: the sequence's first token still moves the logits 300
    tokens later, in a prompt and in decoded tokens; a state that is lost or cleared shows.  (The seed is
    one with which no row's output nearly cancels: its norm would magnify float32's own rounding.)"""
    config = single(kind, _light(2, 24, 20, (0.9999, 1.0)) if kind == "lightning" else _delta(2, 24, 4), vocab=150)
    ids = [149] + [t % 149 for t in random_ids(309, 149, 5)]
    edit = lambda w: plant_memory(w, config, 149)
    d = write_model(tmp_path_factory.getbasetemp(), config, seed=16, dtype=STORE[dtype], edit=edit)
    w = weights64(d)
    want = P.forward(config, w, ids)
    other = [7] + ids[1:]
    moved = (P.forward(config, w, other)[300:] - want[300:]).abs().max() / want[300:].abs().max()
    assert float(moved) > 4 * BUDGET[dtype], float(moved)
    eng = engine_for(d, dtype)
    slot = eng.alloc_slot()
    got = feed(eng, slot, ids, [300])
    close(got[300:], want[300:], dtype, kind + ", the last rows")
    close(got, want, dtype, kind)
    eng.free_slot(slot)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(tmp_path_factory, dtype):
    """A prompt of 20 tokens, then 280 tokens one by one (over pages, windows and the ring, through
    decode graphs)."""
    d = write_model(tmp_path_factory.getbasetemp(), ODD, seed=12, dtype=STORE[dtype])
    eng = engine_for(d, dtype, step_rows=16)
    ids = random_ids(300, ODD["vocab"], 41)
    slot = eng.alloc_slot()
    close(feed(eng, slot, ids, [20]), P.forward(ODD, weights64(d), ids), dtype)
    eng.free_slot(slot)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_engine(tmp_path_factory, dtype):
    """`Engine.generate` (the scheduler's batches, decode graphs, the sampler's arg-max): four
    prompts of unequal lengths with room for two at a time, against the plain model's greedy
    tokens; in bfloat16 a close call may differ, after which the texts part."""
    d = write_model(tmp_path_factory.getbasetemp(), MIXED, seed=7, dtype=STORE[dtype])
    w = weights64(d)
    eng = engine_for(d, dtype, max_batch=2, poison_freed=False)
    prompts = [random_ids(n, MIXED["vocab"], 5 + n) for n in (3, 40, 66, 9)]
    got = eng.generate(prompts, max_new_tokens=12)
    same = 0
    for p, g in zip(prompts, got):
        want = P.generate_greedy(MIXED, w, p, 12)
        assert len(g) == 12
        if dtype == "float32":
            assert g == want
        same += sum(1 for x, y in zip(g, want) if x == y) >= 6
    assert same >= 3
    portions = eng.generate(prompts, max_new_tokens=12, max_step_tokens=16)
    if dtype == "float32":
        assert portions == got


def test_the_command_line_and_the_trace_replay(tmp_path):
    """`bin/chat` with token-id prompts, greedy, names the design by `--type`; `bin/trace_run`
    replays two requests that start together and go on by one token."""
    import subprocess
    import sys
    import numpy as np
    d = write_model(tmp_path, ODD, seed=14, dtype=torch.float32)
    w = weights64(d)
    ids = random_ids(9, ODD["vocab"], 2)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "chat"), "-m", d, "-d", "float32", "--temp", "0",
                        "-n", "5", "--prompt-ids", " ".join(map(str, ids)), "-c", "64", "--type", "febivik"],
                       capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr
    assert [int(t) for t in r.stdout.split()] == P.generate_greedy(ODD, w, ids, 5)
    a, b = random_ids(70, ODD["vocab"], 4), random_ids(5, ODD["vocab"], 6)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:68], "want": [0, 67]},
                                     {"id": "b", "tokens": b[:3], "want": [2]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[68:69], "want": []},
                                     {"id": "b", "tokens": b[3:4], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[69:], "want": [0]},
                                     {"id": "b", "tokens": b[4:], "want": [0]}], "end": ["a", "b"]}]
    out = tmp_path / "out"
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", d, "--dtype", "float32",
                        "--out", str(out), "--max-tokens", "128"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    wa, wb = P.forward(ODD, w, a), P.forward(ODD, w, b)
    V = ODD["vocab"]
    got = {i: torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, V)) for i in range(3)}
    close(got[0], torch.stack([wa[0], wa[67], wb[2]]), "float32")
    close(got[1], wb[3:4], "float32")
    close(got[2], torch.stack([wa[69], wb[4]]), "float32")


def test_a_conversation_in_one_slot(tmp_path):
    """`Engine.session`: the turns of a conversation go on from what the slot holds (keys and
    values, states) by several tokens."""
    d = write_model(tmp_path, MIXED, seed=17)
    w = weights64(d)
    eng = engine_for(d, "float32")
    first = random_ids(6, MIXED["vocab"], 54)
    with eng.session(stop_token_ids=[]) as chat:
        a1 = chat.say(first, max_new_tokens=4)
        assert a1 == P.generate_greedy(MIXED, w, first, 4)
        turn = random_ids(5, MIXED["vocab"], 77)
        a2 = chat.say(turn, max_new_tokens=3)
        assert a2 == P.generate_greedy(MIXED, w, first + a1 + turn, 3)
    eng.cache.check()


# ------------------------------------------------------------------ kernels alone, against their plain torch stand-ins
def _near(got, want, tol=2e-5):
    want = want.double()
    assert float((got.double().cpu() - want).abs().max()) <= tol * max(1.0, float(want.abs().max()))


def _packed(lens, slots):
    cu = torch.tensor([0] + list(torch.tensor(lens).cumsum(0)), dtype=torch.int32)
    row_slot = torch.tensor([s for n, s in zip(lens, slots) for _ in range(n)], dtype=torch.int32)
    return cu, torch.tensor(slots, dtype=torch.int32), row_slot


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_pass_between_sublayers_against_plain_torch(dtype):
    """The sublayer's own norm (RMS or layer norm, or none), the add, and the rows themselves or their
    norm; all rows or some; widths in and out of the vector path."""
    from inferllm_amd.kernels import ops
    g = torch.Generator().manual_seed(3)
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    for T, E in ((5, 90), (1, 4096), (33, 7), (3, 8192), (2, 1030), (4, 256)):
        a = (torch.randn(T, E, generator=g) * 3 + 0.7).to(dtype)
        pw, pb, w, b = ((torch.randn(E, generator=g) + 1).to(dtype) for _ in range(4))
        x, idx = torch.randn(T, E, generator=g), torch.tensor([T - 1, 0], dtype=torch.int32)
        for post in (None, "plain", "rms", "layer", "layer, no bias"):
            for kind, rows, out_dtype in ((None, None, dtype), ("layer", None, dtype), ("layer", idx, dtype),
                                          ("rms", idx, torch.float32), (None, None, None)):
                def make(move):
                    if post is None or post == "plain":
                        return None if post is None else move(a)
                    bias = move(pb) if post == "layer" else None
                    return ops.PostNormed(move(a), move(pw), 1e-5, 0.7, post.split(",")[0], bias)
                cpu, gpu = (lambda t: t), (lambda t: t.cuda())
                x_want, x_got = x.clone(), x.cuda()
                args = lambda move: (kind, move(w) if kind else None, move(b) if kind == "layer" else None, 2e-5, out_dtype,
                                     move(rows) if rows is not None else None)
                want = R.post_add_norm(x_want, make(cpu), *args(cpu))
                got = ops.post_add_norm(x_got, make(gpu), *args(gpu))
                if out_dtype is not None:
                    _near(got, want, tol)
                _near(x_got, x_want, 1e-5)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_activations_without_a_gate_against_plain_torch(dtype):
    from inferllm_amd.kernels import ops
    g = torch.Generator().manual_seed(4)
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    for shape in ((3, 40), (7, 9), (1, 1), (64, 1024)):
        x = (torch.randn(*shape, generator=g) * 3).to(dtype)
        par = torch.tensor([0.7, 1.9])
        _near(ops.xielu(x.cuda(), par.cuda()), R.xielu(x, par), tol)
        _near(ops.relu_squared(x.cuda()), R.relu_squared(x), tol)
        _near(ops.tanh_columns(x.cuda(), shape[1] // 2, shape[1] - shape[1] // 2),
              R.tanh_columns(x, shape[1] // 2, shape[1] - shape[1] // 2), 1e-5)
    small = torch.tensor([[-1e-3, 1e-4, -30.0, -100.0, 0.0, 50.0]]).to(dtype)
    _near(ops.xielu(small.cuda(), par.cuda()), R.xielu(small, par), tol)


@pytest.mark.parametrize("matrix_cores", [1, 2, 0])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_windows_with_kept_tokens_against_plain_torch(dtype, matrix_cores):
    """Biases, weighted norms a head, rotation and the store into a line with kept pages and a ring
    (rows that later rows overwrite are left out); then rows over the step's own keys, rows and
    single tokens over the cache, on the matrix cores and on the vector units, one and several
    ranges of keys; more kept tokens than a page, kept tokens within the window."""
    from inferllm_amd.kernels import ops
    from inferllm_amd.parts.position import rotary_table
    ops._lib().illm_set_attn_cap_mfma(matrix_cores)
    try:
        g = torch.Generator().manual_seed(6)
        tol = 1e-5 if dtype == torch.float32 else 2e-2
        for nh, nkv, dk, dv, window, keep, kept, ring, rot in ((6, 2, 20, 12, 37, 3, 1, 2, 8), (4, 4, 64, 40, 64, 70, 2, 3, 64),
                                                               (5, 1, 36, 130, 9, 1, 1, 2, 0), (8, 2, 128, 128, 100, 130, 3, 4, 32)):
            lens, slots, page = [450, 3, 1, 64], [1, 3, 0, 2], 64
            T, per = sum(lens), kept + ring
            table = torch.randperm(4 * per, generator=g).view(4, per).to(torch.int32)
            cu, seq_slot, row_slot = _packed(lens, slots)
            row_pos = torch.tensor([i for n in lens for i in range(n)], dtype=torch.int32)
            slot_len = torch.zeros(5, dtype=torch.int32)
            for s, n in zip(slots, lens):
                slot_len[s] = n
            k_off, v_off = nh * dk, (nh + nkv) * dk
            rows = torch.randn(T, v_off + nkv * dv + 4, generator=g).to(dtype)
            bias = torch.randn(v_off + nkv * dv, generator=g)
            qw, kw = ((torch.randn(dk, generator=g) * 0.3 + 1).to(dtype) for _ in range(2))
            cs = rotary_table(77.0, rot, 600, "cpu", {"factor": 2.0}) if rot else None
            kc, vc = (torch.zeros(4 * per, nkv, page, n).to(dtype) for n in (dk, dv))
            r_want, kc_want, vc_want = rows.clone(), kc.clone(), vc.clone()
            R.qk_rotate_store(r_want, k_off, v_off, cs, rot, 0, False, 1e-5, row_pos, row_slot, kc_want, vc_want, table,
                              page, ring, nh, nkv, dk, dv, bias=bias, q_weight=qw, k_weight=kw, kept=kept)
            r_got, kc_got, vc_got = rows.cuda(), kc.cuda(), vc.cuda()
            tb, cuG, ssG, slG = table.cuda(), cu.cuda(), seq_slot.cuda(), row_slot.cuda()
            ops.qk_rotate_store(r_got, k_off, v_off, cs.cuda() if rot else None, rot, 0, False, 1e-5, row_pos.cuda(), slG,
                                kc_got, vc_got, tb, page, ring, nh, nkv, dk, dv, bias=bias.cuda(), q_weight=qw.cuda(),
                                k_weight=kw.cuda(), slot_len=slot_len.cuda(), kept=kept)
            # (what lies in the ring's last page behind the sequence's end is of no use to anyone)
            last = [table[1, kept + ((450 - 1) // 64 - kept) % ring]]
            for got, want in ((kc_got, kc_want), (vc_got, vc_want)):
                got, want = got.cpu().clone(), want.clone()
                got[last, :, 450 % 64:], want[last, :, 450 % 64:] = 0, 0
                _near(got, want, tol)
            _near(r_got, r_want, tol)
            starts = torch.zeros(4, dtype=torch.int32)
            own = (k_off, v_off)
            want = R.attn_cap_rows(r_want, cu, seq_slot, starts, kc_want, vc_want, table, page, ring, 4, 450, nh, nkv, dk,
                                   dv, 0.3, 0.0, window, keep=keep, kept=kept, own=own)
            r_in, kc_in, vc_in = r_want.cuda(), kc_want.cuda(), vc_want.cuda()
            got = ops.attn_cap_rows(r_in, cuG, ssG, starts.cuda(), kc_in, vc_in, tb, page, ring, 4, 450, nh, nkv, dk, dv,
                                    0.3, 0.0, window, keep=keep, kept=kept, own=own)
            _near(got, want, tol)
            # the sequences' last rows again over the cache, as a portion and as single tokens
            n2 = [2, 1, 1, 2]
            at = [int(cu[b + 1]) - n + i for b, n in enumerate(n2) for i in range(n)]
            cu2 = torch.tensor([0, 2, 3, 4, 6], dtype=torch.int32)
            start2 = torch.tensor([448, 2, 0, 62], dtype=torch.int32)
            got = ops.attn_cap_rows(r_want[at].cuda(), cu2.cuda(), ssG, start2.cuda(), kc_in, vc_in, tb, page, ring, 4, 2, nh,
                                    nkv, dk, dv, 0.3, 0.0, window, keep=keep, kept=kept)
            _near(got, want[at], tol)
            ends = torch.tensor([int(cu[b + 1]) - 1 for b in range(4)])
            for nsplit in (1, 3):
                got = ops.attn_cap_decode(r_want[ends].cuda(), kc_in, vc_in, tb, page, ring, ssG,
                                          torch.tensor(lens, dtype=torch.int32).cuda(), nh, nkv, dk, dv, 0.3, 0.0, window,
                                          nsplit, keep=keep, kept=kept)
                _near(got, want[ends], tol)
    finally:
        ops._lib().illm_set_attn_cap_mfma(1)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_lightning_kernels_against_plain_torch(dtype):
    """Preparation and scan, the chunks in parallel and the single-token kernel, from states that are
    not zero; lengths on both sides of a chunk's edge; decays of exactly 0 and 1."""
    from inferllm_amd.kernels import ops
    g = torch.Generator().manual_seed(11)
    for H, dk, dv in ((3, 40, 12), (2, 128, 128), (4, 8, 96), (1, 100, 68), (2, 10, 14), (2, 132, 40), (5, 16, 33)):
        decay = torch.tensor([0.97, 0.0, 1.0, 0.5, 0.9995][:H])
        offs = (4, 4 + H * dk, 4 + 2 * H * dk)
        for lens in ([150, 3, 64, 65, 1], [1, 1, 1], [63, 20], [129]):
            T = sum(lens)
            cu, seq_slot, row_slot = _packed(lens, [4, 0, 2, 5, 1][:len(lens)])
            width = -(-(offs[2] + H * dv + 3) // 4) * 4
            U = torch.randn(T, width, generator=g).to(dtype)
            state = torch.randn(6, H, dk, dv, generator=g)
            s_want = state.clone()
            want = R.lightning_chunks(U, *offs, decay, s_want, cu, seq_slot, len(lens), max(lens), H, dk, dv)
            ways = ["scan"]
            if ops.lightning_chunks_fits(U, *offs, dk, dv):
                ways.append("chunks")
            if max(lens) == 1:
                ways.append("step")
            for way in ways:
                s_got, Ug, dG = state.cuda(), U.cuda(), decay.cuda()
                if way == "scan":
                    ins = ops.lightning_prepare(Ug, *offs, dG, H, dk, dv)
                    o = ops.delta_scan(*ins, s_got, cu.cuda(), seq_slot.cuda(), len(lens), max(lens), correct=False)
                elif way == "chunks":
                    o = ops.lightning_chunks(Ug, *offs, dG, s_got, cu.cuda(), seq_slot.cuda(), len(lens), max(lens), H, dk, dv)
                else:
                    o = ops.lightning_step(Ug, *offs, dG, s_got, row_slot.cuda(), H, dk, dv)
                _near(o, want, 1e-5); _near(s_got, s_want, 1e-5)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_delta_rule_with_a_removal_vector_against_plain_torch(dtype):
    """Preparation and scan (short and long steps), the chunks and the single-token kernel with its
    low-rank map, from states that are not zero; lengths on both sides of a chunk's edge, decays as
    strong and as weak as they get."""
    from inferllm_amd.kernels import ops
    g = torch.Generator().manual_seed(12)
    rate = 0.6
    for H, d, rank in ((3, 24, 5), (2, 128, 64), (4, 10, 3), (1, 200, 16), (2, 64, 130), (8, 96, 7)):
        n = H * d
        offs = (2, 2 + n, 2 + 2 * n, 2 + 3 * n)
        w1_off = 2 + 4 * n
        a_bias, w0 = torch.randn(n, generator=g), torch.randn(n, generator=g) * 2 - 1
        w0[::5], w0[1::5] = 12.0, -12.0
        w2 = (torch.randn(n, rank, generator=g) / rank ** 0.5).to(dtype)
        for lens in ([70, 3, 16, 1], [1, 1, 1], [5, 2], [64, 31, 33, 32], [257]):
            T = sum(lens)
            cu, seq_slot, row_slot = _packed(lens, [4, 0, 2, 5][:len(lens)])
            U = torch.randn(T, w1_off + rank + 1, generator=g).to(dtype)
            Z = torch.randn(T, n, generator=g)
            state = torch.randn(6, H, d, d, generator=g)
            want_in = R.removal_prepare(U, *offs, a_bias, Z, w0, rate, H, d)
            got_in = ops.removal_prepare(U.cuda(), *offs, a_bias.cuda(), Z.cuda(), w0.cuda(), rate, H, d)
            for a, b in zip(got_in, want_in):
                _near(a, b, 1e-5)
            s_want, s_got = state.clone(), state.cuda()
            want = R.delta_scan(*want_in[:5], s_want, cu, seq_slot, len(lens), max(lens), correct=False, removal=want_in[5])
            o = ops.delta_scan(*got_in[:5], s_got, cu.cuda(), seq_slot.cuda(), len(lens), max(lens), correct=False,
                               removal=got_in[5])
            _near(o, want, 2e-5); _near(s_got, s_want, 2e-5)
            if d <= 128:
                s_got = state.cuda()
                o = ops.removal_chunks(U.cuda(), *offs, a_bias.cuda(), Z.cuda(), w0.cuda(), rate, s_got, cu.cuda(),
                                       seq_slot.cuda(), len(lens), max(lens), H, d)
                _near(o, want, 2e-5); _near(s_got, s_want, 2e-5)
            if max(lens) == 1:
                s_want, s_got = state.clone(), state.cuda()
                want = R.removal_step(U, *offs, a_bias, w1_off, w2, w0, rate, s_want, row_slot, H, d)
                o = ops.removal_step(U.cuda(), *offs, a_bias.cuda(), w1_off, w2.cuda(), w0.cuda(), rate, s_got,
                                     row_slot.cuda(), H, d)
                _near(o, want, 2e-5); _near(s_got, s_want, 2e-5)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_norm_in_parts_with_a_gate_against_plain_torch(dtype):
    from inferllm_amd.kernels import ops
    g = torch.Generator().manual_seed(13)
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    for T, width, groups in ((5, 96, 4), (3, 90, 9), (2, 2048, 1), (1, 1030, 1), (4, 1024, 2), (3, 4096, 32)):
        for off in (3, 8):
            o, w = torch.randn(T, width, generator=g) * 2, (torch.randn(width, generator=g) + 1).to(dtype)
            Z = torch.randn(T, width + off + (5 if off == 3 else 0), generator=g).to(dtype)
            for gate in ("sigmoid", "silu"):
                _near(ops.group_norm_gate(o.cuda(), groups, w.cuda(), Z.cuda(), off, gate, 1e-5, dtype),
                      R.group_norm_gate(o, groups, w, Z, off, gate, 1e-5, dtype), tol)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T", [1, 9, 70, 300])
def test_experts_without_a_gate_against_plain_torch(T, dtype):
    """Routing with a scale on the weights, the grouped squared-ReLU experts (every tile size, sizes in
    and out of the matrix cores' steps) and the weighted sum with an ungated shared expert's rows."""
    from inferllm_amd.kernels import ops
    g = torch.Generator().manual_seed(T)
    tol = 2e-5 if dtype == torch.float32 else 2e-2
    for E, F, n_exp, top in ((64, 96, 4, 2), (128, 64, 3, 3), (90, 30, 7, 2), (256, 32, 5, 1)):
        h = torch.randn(T, E, generator=g).to(dtype)
        wr = torch.randn(n_exp, E, generator=g) * (2.0 / E ** 0.5)
        up = (torch.randn(n_exp, F, E, generator=g) / E ** 0.5).to(dtype)
        down = (torch.randn(n_exp, E, F, generator=g) / F ** 0.5).to(dtype)
        shared = torch.randn(T, E, generator=g).to(dtype)
        idx, wt, _ = R.moe_plan(h, wr, None, top, up, "softmax", 1.7, False)
        g_idx, g_wt, grouped = ops.moe_plan(h.cuda(), wr.cuda(), None, top, up.cuda(), "softmax", 1.7, False)
        assert torch.equal(g_idx.cpu(), idx)
        _near(g_wt, wt, 1e-5)
        y = R.moe_experts(h, idx, up, down, activation="relu_squared")
        g_y = ops.moe_experts(h.cuda(), g_idx, up.cuda(), down.cuda(), grouped, "relu_squared")
        _near(g_y, y, tol)
        _near(ops.moe_combine(h.cuda(), g_idx, g_wt, g_y, n_exp, shared.cuda()), R.moe_combine(h, idx, wt, y, n_exp, shared),
              tol)
