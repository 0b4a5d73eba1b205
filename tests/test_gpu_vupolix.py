"""Vupolix through the engine against the plain model (tests/plain_vupolix.py): every mechanism in a layer of
its own, whole prompts, token-by-token decoding, prompts cut into portions down to two tokens, batches of unequal
requests, slots, pages and states used again, passes of repeated layers, planted keys far away, at page borders
and just inside and just outside a window, in prompts and in decoding and past the end of the cache's ring, the
sink, a memory from far back, long decoding, greedy generation through the engine's own loop, the command line
and the trace replay; and the new kernels alone.  Configurations: tests/vupolix_tiny.py."""
import json
import os

import pytest
import torch

import kernel_refs as R
import plain_vupolix as P
from vupolix_tiny import (CONFIGS, MIXED, ODD, REPEATED, SEEDS, _layer, _left, _model, _moe, _par, _right, _rot, _wkv, plant_key,
                          plant_memory, single, weights64, write_model)
from tiny import random_ids

pytestmark = pytest.mark.gpu

BUDGET = {"float32": 3e-5, "bfloat16": 5e-2}
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
SMALL_LEFT, SMALL_RIGHT = _left(2, 1, 8, 0.4), _right(2, 8, 8, (0.9, 0.7))
TWICE = _model([_layer(_wkv(2, 16, 4)), _layer(_wkv(3, 8, 2))], vocab=200, width=64, eps=1e-6, gain=0.5, logit_scale=1.0,
               loop=(0, 2, 2))
MECHANISMS = {
    "time_mix_small": single(_wkv(3, 10, 2)),
    "time_mix_wider_than_the_model": single(_wkv(3, 32, 7)),
    "time_mix_128": single(_wkv(1, 128, 16)),
    "time_mix_beyond_the_chunks": single(_wkv(2, 132, 5)),
    "attention_grouped_part_rotated": single(_par(_left(6, 3, 16, 0.3, None, _rot(700.0, 6, (2.5, 100, 8.0, 1.0))), SMALL_RIGHT)),
    "attention_all_rotated_one_kv_head": single(_par(_left(5, 1, 24, 0.4, 23, _rot(20000.0, 24)), SMALL_RIGHT)),
    "attention_without_rotation": single(_par(_left(4, 2, 12, 0.4, 33), SMALL_RIGHT)),
    "attention_wide_heads": single(_par(_left(2, 2, 136, 0.1, 40, _rot(100.0, 64, (4.0, 50, 4.0, 1.0))), SMALL_RIGHT)),
    "window_of_one": single(_par(_left(2, 1, 16, 0.9, 1, _rot(9.0, 8)), SMALL_RIGHT)),
    "retention_wide_keys": single(_par(SMALL_LEFT, _right(3, 40, 12, (0.9, 0.5, 0.99), _rot(50.0, 20)))),
    "retention_wide_values": single(_par(SMALL_LEFT, _right(2, 8, 72, (0.97, 0.3)))),
    "retention_sizes_of_two": single(_par(SMALL_LEFT, _right(2, 10, 14, (1.0, 0.0), _rot(30.0, 10)))),
    "retention_beyond_the_chunks": single(_par(SMALL_LEFT, _right(2, 132, 136, (0.9, 0.99), _rot(30.0, 66)))),
    "experts_in_groups": single(_wkv(2, 8, 2), _moe(40, 12, 3, (4, 2), 52)),
    "experts_in_groups_of_one": single(_wkv(2, 8, 2), _moe(40, 4, 2, (4, 3))),
    "experts_in_one_group": single(_wkv(2, 8, 2), _moe(24, 5, 1, (1, 1), 20)),
    "experts_without_groups": single(_wkv(2, 8, 2), _moe(32, 5, 2, None, 36)),
    "experts_on_the_matrix_cores": single(_wkv(2, 8, 2), _moe(64, 8, 2, (2, 1), 96)),
    "repeated_layers": TWICE,
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(MECHANISMS))
def test_mechanism_alone_prompt_and_tokens(tmp_path_factory, name, dtype):
    """A model of one layer (or two, twice) that has the mechanism: a prompt of 70 tokens, then 10 single tokens."""
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
    d = write_model(tmp_path_factory.getbasetemp(), config, seed=SEEDS[name], dtype=STORE[dtype])
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
    d = write_model(tmp_path_factory.getbasetemp(), MIXED, seed=SEEDS["MIXED"], dtype=STORE[dtype])
    eng = engine_for(d, dtype)
    ids = random_ids(140, MIXED["vocab"], 23)
    want = P.forward(MIXED, weights64(d), ids)
    slot = eng.alloc_slot()
    close(feed(eng, slot, ids if cuts else ids[:45], cuts), want if cuts else want[:45], dtype, str(cuts))
    eng.free_slot(slot)
    eng.cache.check()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cuts", [[400], [150, 152, 290, 400], [60, 61, 320], [1, 200]])
def test_prompts_longer_than_the_ring(tmp_path_factory, cuts, dtype):
    """400 tokens and more through a ring of a few pages: whole (keys and values then come from the step's own
    rows), in portions (cut further by the step function where they would write round the ring) and token
    by token."""
    d = write_model(tmp_path_factory.getbasetemp(), ODD, seed=SEEDS["ODD"], dtype=STORE[dtype])
    eng = engine_for(d, dtype, step_rows=32)
    assert all(g.ring for g in eng.cache.groups)
    n = 410 if cuts[-1] == 400 else cuts[-1] + 20
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
    d = write_model(tmp_path_factory.getbasetemp(), ODD, seed=SEEDS["ODD"], dtype=STORE[dtype])
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
    d = write_model(tmp_path_factory.getbasetemp(), MIXED, seed=SEEDS["MIXED"], dtype=STORE[dtype])
    w = weights64(d)
    eng = engine_for(d, dtype, max_batch=2, max_tokens=384, max_seq_len=256, step_rows=16)
    for turn in range(3):
        reqs = [random_ids(n, MIXED["vocab"], 100 * turn + n) for n in (100 + turn * 30, 40 + turn)]
        slots = [eng.alloc_slot() for _ in reqs]
        out = eng.step([StepEntry(s, r[:-3], list(range(len(r) - 3))) for s, r in zip(slots, reqs)])
        got = [[out[:len(reqs[0]) - 3].clone()], [out[len(reqs[0]) - 3:].clone()]]
        for t in (3, 2, 1):
            out = eng.step([StepEntry(s, [r[-t]], [0]) for s, r in zip(slots, reqs)])
            got[0].append(out[:1].clone()); got[1].append(out[1:].clone())
        for i, r in enumerate(reqs):
            close(torch.cat(got[i]), P.forward(MIXED, w, r), dtype, f"pass {turn} request {i}")
        for s in slots:
            eng.free_slot(s)
        eng.cache.check()


@pytest.mark.parametrize("kind", ["wkv", "retention"])
def test_state_starts_at_zero_in_a_slot_used_before(tmp_path_factory, kind):
    """State, and the row that the token shift keeps, are cleared when a slot is handed out: the same request
    twice in the same slot gives the same bits, with another request between."""
    from inferllm_amd import StepEntry
    config = single(_wkv(3, 16, 4) if kind == "wkv" else _par(SMALL_LEFT, _right(2, 16, 24, (0.99, 0.7))), _moe(32, 4, 2))
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
    d = write_model(tmp_path_factory.getbasetemp(), MIXED, seed=SEEDS["MIXED"], dtype=torch.float32)
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


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_decoding_batches_of_every_size(tmp_path_factory, dtype):
    """1, 5, 20 and 70 sequences decoded together (products of few rows, of up to 128 from the decode copies, the
    graphs' filling rows), against each alone."""
    from inferllm_amd import StepEntry
    d = write_model(tmp_path_factory.getbasetemp(), REPEATED, seed=SEEDS["REPEATED"], dtype=STORE[dtype])
    w = weights64(d)
    eng = engine_for(d, dtype, max_batch=72, max_tokens=72 * 64, max_seq_len=64)
    reqs = [random_ids(4 + (7 * i) % 23, REPEATED["vocab"], i) for i in range(70)]
    want = [P.forward(REPEATED, w, r) for r in reqs]
    for n in (1, 5, 20, 70):
        slots = [eng.alloc_slot() for _ in range(n)]
        eng.step([StepEntry(s, r[:-3], []) for s, r in zip(slots, reqs)])
        rows = [eng.step([StepEntry(s, [r[t]], [0]) for s, r in zip(slots, reqs)]).clone() for t in (-3, -2, -1)]
        got = torch.stack(rows, 1).reshape(3 * n, -1)
        close(got, torch.cat([x[-3:] for x in want[:n]]), dtype, f"{n} sequences")
        for s in slots:
            eng.free_slot(s)


# ------------------------------------------------------------------ far keys, window edges, the sink
def _planted(tmp_path_factory, config, dtype, n, query_at, key_at, seed=8, more=None):
    KEY, QUERY = 250, 251
    ids = [t % 250 for t in random_ids(n, 250, 31)]
    ids[key_at] = KEY
    if query_at != key_at:
        ids[query_at] = QUERY

    def edit(w):
        plant_key(w, config, KEY, QUERY if query_at != key_at else KEY)
        if more is not None:
            more(w)
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


def _moved(wrong, want, at):
    return float((wrong[at] - want[at]).abs().max() / want[at].abs().max())


PLANT_ROT, PLANT_RIGHT = _rot(10000.0, 8, (2.0, 300, 8.0, 1.0)), _right(2, 8, 12, (0.9, 0.6))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("query_at, key_at", [(399, 0), (399, 3), (300, 63), (300, 64), (257, 128), (1, 0), (5, 5)])
def test_a_planted_key_far_back_under_full_attention(tmp_path_factory, query_at, key_at, dtype):
    """One position's key is made to stand out for one query position hundreds of tokens later (at
    the sequence's first tokens, on both sides of page borders), in a prompt and as a decoded
    token; the same sequence without the key token gives logits far from the right ones."""
    config = single(_par(_left(4, 2, 16, 1.0, None, PLANT_ROT), PLANT_RIGHT), _moe(40, 4, 2), vocab=260)
    d, ids = _planted(tmp_path_factory, config, dtype, 400, query_at, key_at)
    w = weights64(d)
    want = P.forward(config, w, ids)
    assert _moved(P.forward(config, w, ids[:key_at] + [7] + ids[key_at + 1:]), want, query_at) > 4 * BUDGET[dtype]
    _prompt_and_decoded(d, dtype, ids, want, query_at)


WINDOW = 37


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("step_rows", [16, 512])             # the ring wraps within the sequence, or never does
@pytest.mark.parametrize("query_at, key_at", [
    (110, 74), (110, 73),          # the window's last position, and the one beyond it
    (100, 64), (100, 63),          # the same on both sides of the page border at 64
    (293, 257), (293, 256), (164, 128), (164, 127),
    (36, 0), (37, 0), (40, 3), (40, 4), (1, 0),             # the sequence's first tokens
])
def test_a_planted_key_at_the_edges_of_a_window(tmp_path_factory, query_at, key_at, step_rows, dtype):
    """A key at the window's far edge is seen, one position further it is not.  A window that is one off moves
    the logits by far more than the budget."""
    config = single(_par(_left(4, 2, 16, 1.0, WINDOW, PLANT_ROT), PLANT_RIGHT), _moe(40, 4, 2), vocab=260)
    d, ids = _planted(tmp_path_factory, config, dtype, 300, query_at, key_at)
    w = weights64(d)
    want = P.forward(config, w, ids)
    dist = query_at - key_at
    wrong = (P.forward(config, w, ids[:key_at] + [7] + ids[key_at + 1:]) if dist < WINDOW - 1
             else P.forward(config, w, ids, edge_shift=-1 if dist < WINDOW else 1))
    assert _moved(wrong, want, query_at) > 4 * BUDGET[dtype]
    _prompt_and_decoded(d, dtype, ids, want, query_at, step_rows=step_rows)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("size, step_rows", [(None, 512), (37, 16), (1, 16)])
def test_the_sink_counts(tmp_path_factory, size, step_rows, dtype):
    """Sinks from far below to far above the scores, one a head, in prompts (over the cache and over the step's
    own rows) and in decoding; without them the logits are far from the right ones."""
    config = single(_par(_left(6, 2, 16, 0.5, size, PLANT_ROT), PLANT_RIGHT))

    def edit(w):
        w["l0.mix.left.sink"][:] = torch.tensor([-30.0, 1.0, 3.0, 6.0, 0.0, 150.0])
        w["l0.mix.right.out"][:] *= 0.2
    d = write_model(tmp_path_factory.getbasetemp(), config, seed=31, dtype=STORE[dtype], edit=edit)
    w = weights64(d)
    ids = random_ids(150, config["vocab"], 3)
    want = P.forward(config, w, ids)
    wrong = P.forward(config, w, ids, sink_on=False)
    assert float(((wrong - want).abs().amax(-1) / want.abs().max()).median()) > 3 * BUDGET[dtype]
    eng = engine_for(d, dtype, step_rows=step_rows)
    for cuts in ([140], [3, 60, 62, 140], [1, 90]):
        slot = eng.alloc_slot()
        close(feed(eng, slot, ids, cuts), want, dtype, str(cuts))
        eng.free_slot(slot)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["wkv", "retention"])
def test_a_memory_from_far_back(tmp_path_factory, kind, dtype):
    """A recurrent layer that hardly forgets: the sequence's first token still moves the logits 300
    tokens later, in a prompt and in decoded tokens; a state that is lost or cleared shows."""
    config = single(_wkv(2, 24, 4) if kind == "wkv" else _par(SMALL_LEFT, _right(2, 24, 20, (0.9999, 1.0), _rot(10000.0, 4))),
                    vocab=150)
    ids = [149] + [t % 149 for t in random_ids(309, 149, 5)]
    d = write_model(tmp_path_factory.getbasetemp(), config, seed=16, dtype=STORE[dtype],
                    edit=lambda w: plant_memory(w, config, 149))
    w = weights64(d)
    want = P.forward(config, w, ids)
    moved = (P.forward(config, w, [7] + ids[1:])[300:] - want[300:]).abs().max() / want[300:].abs().max()
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
    d = write_model(tmp_path_factory.getbasetemp(), ODD, seed=SEEDS["ODD"], dtype=STORE[dtype])
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
    d = write_model(tmp_path_factory.getbasetemp(), MIXED, seed=SEEDS["MIXED"], dtype=STORE[dtype])
    w = weights64(d)
    eng = engine_for(d, dtype, max_batch=2, poison_freed=False)
    prompts = [random_ids(n, MIXED["vocab"], 5 + n) for n in (3, 40, 66, 9)]
    got = eng.generate(prompts, max_new_tokens=10)
    same = 0
    for p, g in zip(prompts, got):
        want = P.generate_greedy(MIXED, w, p, 10)
        assert len(g) == 10
        if dtype == "float32":
            assert g == want
        same += sum(1 for x, y in zip(g, want) if x == y) >= 5
    assert same >= 3
    portions = eng.generate(prompts, max_new_tokens=10, max_step_tokens=16)
    if dtype == "float32":
        assert portions == got


def test_the_command_line_and_the_trace_replay(tmp_path):
    """`bin/chat` with token-id prompts, greedy, names the design by `--type`; `bin/trace_run`
    replays two requests that start together and go on by one token."""
    import subprocess
    import sys
    import numpy as np
    d = write_model(tmp_path, ODD, seed=SEEDS["ODD"], dtype=torch.float32)
    w = weights64(d)
    ids = random_ids(9, ODD["vocab"], 2)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "chat"), "-m", d, "-d", "float32", "--temp", "0",
                        "-n", "5", "--prompt-ids", " ".join(map(str, ids)), "-c", "64", "--type", "vupolix"],
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
    values, states, the token shift's row) by several tokens."""
    d = write_model(tmp_path, MIXED, seed=SEEDS["MIXED"])
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
def test_pass_with_a_pair_added_rows_and_a_shift_against_plain_torch(dtype):
    """Two outputs under norms of their own, one output, or none; rows added as well; the normed rows themselves (all
    or some) or their mixes with the rows before; widths in and out of the vector path, of one group of four columns a
    thread and of several."""
    from inferllm_amd.kernels import ops
    g = torch.Generator().manual_seed(3)
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    for T, E in ((5, 90), (1, 4096), (33, 7), (3, 8192), (2, 1030), (4, 256), (2, 2048), (1, 6000)):
        rnd = lambda *s: torch.randn(*s, generator=g)
        a, b = (rnd(T, E) * 3).to(dtype), (rnd(T, E) * 0.2).to(dtype)
        wa, wb, pw, w = ((rnd(E) + 1).to(dtype) for _ in range(4))
        x, plus, mu = rnd(T, E), rnd(T, E), rnd(5, E)
        slots = torch.randperm(T + 2, generator=g)[:T].to(torch.int32)
        tail, idx = rnd(T + 2, 1, E).to(dtype), torch.tensor([T - 1, 0], dtype=torch.int32)
        for what in ("pair", "one", "none"):
            for added in (True, False):
                for mode in ("rows", "some rows", "mixes"):
                    if what == "none" and added:
                        continue
                    def run(ops_or_ref, move, x_in, tail_in):
                        post = None
                        if what != "none":
                            y = (ops.NormedPair(move(a), move(wa), move(b), move(wb), 2e-5, 0.5) if what == "pair"
                                 else move(a))
                            post = ops.PostNormed(y, move(pw), 1e-5, 0.7, plus=move(plus) if added else None)
                        return ops_or_ref.post_add_rmsnorm(
                            x_in, post, move(w), 3e-5, dtype, move(idx) if mode == "some rows" else None,
                            shift=(move(mu), tail_in, move(slots)) if mode == "mixes" else None)
                    x_want, x_got, t_want, t_got = x.clone(), x.cuda(), tail.clone(), tail.cuda()
                    want = run(R, lambda t: t, x_want, t_want)
                    got = run(ops, lambda t: t.cuda(), x_got, t_got)
                    assert got.shape == want.shape
                    _near(got, want, tol)
                    _near(x_got, x_want, 1e-5)
                    _near(t_got, t_want, tol)
        pair = ops.NormedPair(a.cuda(), wa.cuda(), b.cuda(), wb.cuda(), 2e-5, 0.5)
        _near(ops.PostNormed(pair, pw.cuda(), 1e-5, 0.7, plus=plus.cuda()).tensor(),
              R._left_to_add(ops.PostNormed(ops.NormedPair(a, wa, b, wb, 2e-5, 0.5), pw, 1e-5, 0.7, plus=plus)), 1e-5)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_embedding_under_a_norm_and_the_copy_against_plain_torch(dtype):
    from inferllm_amd.kernels import ops
    g = torch.Generator().manual_seed(5)
    for V, E in ((30, 90), (7, 2048), (100, 33)):
        table, w = torch.randn(V, E, generator=g).to(dtype), (torch.randn(E, generator=g) + 1).to(dtype)
        tokens = torch.randint(0, V, (9,), generator=g).to(torch.int32)
        out = ops.embed_norm(tokens.cuda(), table.cuda(), w.cuda(), 1e-5, 0.3)
        _near(out, R.embed_norm(tokens, table, w, 1e-5, 0.3), 1e-5)
        assert torch.equal(ops.copy_rows(out), out)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_token_mixes_against_plain_torch(dtype):
    """Rows of several sequences, from kept rows that are not zero; the kept rows moved on by single tokens in the
    same launch and by longer steps afterwards."""
    from inferllm_amd.kernels import ops
    g = torch.Generator().manual_seed(6)
    tol = 1e-6 if dtype == torch.float32 else 1e-2
    for E in (90, 96, 2048):
        for lens in ([5, 1, 3, 2], [1, 1, 1]):
            cu, seq_slot, row_slot = _packed(lens, [4, 0, 2, 5][:len(lens)])
            h, mu = torch.randn(sum(lens), E, generator=g).to(dtype), torch.randn(5, E, generator=g)
            tail = torch.randn(6, 1, E, generator=g).to(dtype)
            single_tokens = max(lens) == 1
            t_want, t_got = tail.clone(), tail.cuda()
            want = R.token_mix(h, mu, t_want, row_slot, single_tokens)
            got = ops.token_mix(h.cuda(), mu.cuda(), t_got, row_slot.cuda(), single_tokens)
            if not single_tokens:
                R.short_conv_tail(h, 0, t_want, cu, seq_slot, len(lens), 2)
                ops.short_conv_tail(h.cuda(), 0, t_got, cu.cuda(), seq_slot.cuda(), len(lens), 2)
            _near(got, want, tol)
            assert torch.equal(t_got.cpu(), t_want)


def test_products_whose_parts_read_rows_of_their_own():
    """One launch for few rows (with and without the decode copy), one or several for more, one product a part for
    everything else; parts in and out of the launches' steps."""
    from inferllm_amd.kernels import ops
    g = torch.Generator().manual_seed(7)
    for dtype in (torch.bfloat16, torch.float32):
        tol = 2e-2 if dtype == torch.bfloat16 else 1e-5
        for K, ends in ((128, (64, 128, 192, 256, 272)), (192, (96, 192, 288, 384, 400)), (90, (30, 60, 95)),
                        (256, (512, 1024, 1536, 2048, 2112)), (64, (48, 96))):
            w = (torch.randn(ends[-1], K, generator=g) / K ** 0.5).to(dtype)
            for copies in (False, True):
                wg = ops.decode_weight(w.cuda(), "plain", copies)
                for M in (1, 9, 16, 17, 40, 64, 100, 128, 150):
                    planes = torch.randn(len(ends), M, K, generator=g).to(dtype)
                    got = ops.linear_parts(planes.cuda(), wg, ends)
                    want = R.linear_parts(planes.double(), w.double(), ends)
                    assert len(got) == len(ends)
                    for x, y in zip(got, want):
                        assert x.shape == y.shape
                        _near(x, y, tol)


@pytest.mark.parametrize("matrix_cores", [1, 2, 0])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_attention_with_a_sink_over_its_own_keys_against_plain_torch(dtype, matrix_cores):
    """Rotation and the store with values that are the unrotated keys; then rows over the step's own keys (values in
    rows of their own), rows and single tokens over the cache, on the matrix cores and on the vector units, one and
    several ranges of keys, with a ring and without; sinks from far below to far above every score."""
    from inferllm_amd.kernels import ops
    from inferllm_amd.parts.position import rotary_table
    ops._lib().illm_set_attn_cap_mfma(matrix_cores)
    try:
        g = torch.Generator().manual_seed(6)
        tol = 1e-5 if dtype == torch.float32 else 2e-2
        for nh, nkv, d, window, ring, rot in ((6, 2, 20, 37, 2, 8), (4, 4, 64, 64, 3, 64), (5, 1, 132, 9, 2, 0), (8, 2, 128, 0, 0, 32)):
            lens, slots, page = [300, 3, 1, 64], [1, 3, 0, 2], 64
            T, per = sum(lens), ring or 6
            table = torch.randperm(4 * per, generator=g).view(4, per).to(torch.int32)
            cu, seq_slot, row_slot = _packed(lens, slots)
            row_pos = torch.tensor([i for n in lens for i in range(n)], dtype=torch.int32)
            slot_len = torch.zeros(5, dtype=torch.int32)
            for s, n in zip(slots, lens):
                slot_len[s] = n
            k_off, g_off = nh * d, (nh + nkv) * d
            rows = torch.randn(T, g_off + nh + 8 - (g_off + nh) % 8, generator=g).to(dtype)
            sink = torch.linspace(-40.0, 120.0, nh)[torch.randperm(nh, generator=g)]
            cs = rotary_table(77.0, rot, 600, "cpu") if rot else None
            kc, vc = (torch.zeros(4 * per, nkv, page, d).to(dtype) for _ in range(2))
            r_want, kc_want, vc_want, v_want = rows.clone(), kc.clone(), vc.clone(), torch.zeros(T, nkv * d).to(dtype)
            R.qk_rotate_store(r_want, k_off, 0, cs, rot, 0, False, 1e-5, row_pos, row_slot, kc_want, vc_want, table, page,
                              ring, nh, nkv, d, d, values_from_keys=True, values_out=v_want)
            r_got, kc_got, vc_got, v_got = rows.cuda(), kc.cuda(), vc.cuda(), torch.zeros_like(v_want).cuda()
            tb, cuG, ssG, slG = table.cuda(), cu.cuda(), seq_slot.cuda(), row_slot.cuda()
            ops.qk_rotate_store(r_got, k_off, 0, cs.cuda() if rot else None, rot, 0, False, 1e-5, row_pos.cuda(), slG, kc_got,
                                vc_got, tb, page, ring, nh, nkv, d, d, slot_len=slot_len.cuda() if ring else None,
                                values_from_keys=True, values_out=v_got)
            assert torch.equal(v_got.cpu(), v_want)
            _near(r_got, r_want, tol)
            if not ring:
                _near(kc_got, kc_want, tol); _near(vc_got, vc_want, tol)
            starts = torch.zeros(4, dtype=torch.int32)
            # (over the step's own rows; the cache's ring does not hold the longest sequence)
            args = (4, max(lens), nh, nkv, d, d, 0.3, 0.0, window)
            want = R.attn_cap_rows(r_want, cu, seq_slot, starts, kc_want, vc_want, table, page, ring, *args, gate=r_want,
                                   gate_off=g_off, gate_heads=True, own=(k_off, 0), own_values=v_want, sink=sink)
            r_in, v_in, sG = r_want.cuda(), v_want.cuda(), sink.cuda()
            got = ops.attn_cap_rows(r_in, cuG, ssG, starts.cuda(), kc_got, vc_got, tb, page, ring, *args, gate=r_in,
                                    gate_off=g_off, gate_heads=True, own=(k_off, 0), own_values=v_in, sink=sG)
            _near(got, want, tol)
            # the sequences' last rows again over the cache, as a portion and as single tokens
            n2 = [2, 1, 1, 2]
            at = [int(cu[b + 1]) - n + i for b, n in enumerate(n2) for i in range(n)]
            cu2 = torch.tensor([0, 2, 3, 4, 6], dtype=torch.int32)
            start2 = torch.tensor([298, 2, 0, 62], dtype=torch.int32)
            q2 = r_want[at].cuda()
            got = ops.attn_cap_rows(q2, cu2.cuda(), ssG, start2.cuda(), kc_got, vc_got, tb, page, ring, 4, 2, nh, nkv, d, d, 0.3,
                                    0.0, window, gate=q2, gate_off=g_off, gate_heads=True, sink=sG)
            _near(got, want[at], tol)
            ends = torch.tensor([int(cu[b + 1]) - 1 for b in range(4)])
            q1 = r_want[ends].cuda()
            for nsplit in (1, 3):
                got = ops.attn_cap_decode(q1, kc_got, vc_got, tb, page, ring, ssG, torch.tensor(lens, dtype=torch.int32).cuda(),
                                          nh, nkv, d, d, 0.3, 0.0, window, nsplit, gate=q1, gate_off=g_off, gate_heads=True,
                                          sink=sG)
                _near(got, want[ends], tol)
    finally:
        ops._lib().illm_set_attn_cap_mfma(1)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_retention_kernels_against_plain_torch(dtype):
    """Preparation and scan, the chunks in parallel and the single-token kernel with its rotation, from states that are
    not zero; lengths on both sides of a chunk's edge; decays of exactly 0 and 1; positions that do not start at 0."""
    from inferllm_amd.kernels import ops
    from inferllm_amd.parts.position import rotary_table
    g = torch.Generator().manual_seed(11)
    for H, dk, dv, rot in ((3, 40, 12, 16), (2, 128, 128, 128), (4, 8, 96, 0), (1, 100, 68, 98), (2, 10, 14, 10), (2, 132, 40, 6), (5, 16, 33, 4)):
        decay = torch.tensor([0.97, 0.0, 1.0, 0.5, 0.9995][:H])
        offs = (4, 4 + H * dk, 4 + 2 * H * dk)
        cs = rotary_table(50.0, rot, 400, "cpu") if rot else None
        for lens in ([150, 3, 64, 65, 1], [1, 1, 1], [63, 20], [129]):
            T = sum(lens)
            cu, seq_slot, row_slot = _packed(lens, [4, 0, 2, 5, 1][:len(lens)])
            row_pos = torch.tensor([7 * b + i for b, n in enumerate(lens) for i in range(n)], dtype=torch.int32)
            width = -(-(offs[2] + H * dv + 3) // 4) * 4
            U = torch.randn(T, width, generator=g).to(dtype)
            state = torch.randn(6, H, dk, dv, generator=g)
            s_want = state.clone()
            ins_want = R.retention_prepare(U, *offs, decay, cs, rot, 0.3, row_pos, H, dk, dv)
            want = R.delta_scan(*ins_want, s_want, cu, seq_slot, len(lens), max(lens), correct=False)
            ways = ["scan"] + (["chunks"] if ops.retention_chunks_fits(U, offs[2], dk, dv) else []) + (["step"] if max(lens) == 1 else [])
            for way in ways:
                s_got, Ug, dG, cG, pG = state.cuda(), U.cuda(), decay.cuda(), cs.cuda() if rot else None, row_pos.cuda()
                rest = (cu.cuda(), seq_slot.cuda(), len(lens), max(lens))
                if way == "scan":
                    ins = ops.retention_prepare(Ug, *offs, dG, cG, rot, 0.3, pG, H, dk, dv)
                    for x, y in zip(ins, ins_want):
                        _near(x, y, 1e-5)
                    o = ops.delta_scan(*ins, s_got, *rest, correct=False)
                elif way == "chunks":
                    qn, kn = ops.retention_prepare(Ug, *offs, dG, cG, rot, 0.3, pG, H, dk, dv, scan=False)
                    o = ops.retention_chunks(qn, kn, Ug, offs[2], dG, s_got, *rest, H, dk, dv)
                else:
                    o = ops.retention_step(Ug, *offs, dG, cG, rot, 0.3, pG, s_got, row_slot.cuda(), H, dk, dv)
                _near(o, want, 1e-5); _near(s_got, s_want, 1e-5)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_time_mix_kernels_against_plain_torch(dtype):
    """Preparation and scan (short and long steps), the chunks and the single-token kernel with its low-rank map, from
    states that are not zero; lengths on both sides of a chunk's and a sub-block's edge; channels that keep everything,
    that forget everything within a token, and that change from the one to the other; rows that are columns of wider
    rows."""
    from inferllm_amd.kernels import ops
    g = torch.Generator().manual_seed(12)
    for H, d, rank in ((3, 24, 5), (2, 128, 64), (4, 10, 3), (1, 200, 16), (2, 64, 130), (8, 96, 7), (2, 32, 8)):
        n = H * d
        w0, bonus = torch.randn(n, generator=g) * 2 - 1, torch.randn(n, generator=g)
        w0[::5], w0[1::5] = 6.0, -12.0
        w2 = (torch.randn(n, rank, generator=g) / rank ** 0.5).to(dtype)
        for lens in ([70, 3, 16, 1], [1, 1, 1], [5, 2], [64, 31, 33, 32], [257], [17, 15, 48, 49]):
            T = sum(lens)
            cu, seq_slot, row_slot = _packed(lens, [4, 0, 2, 5][:len(lens)])
            U = torch.randn(T, 3 * n + rank + 4 - rank % 4, generator=g).to(dtype)
            cols = lambda t: (t[:, :n], t[:, n:2 * n], t[:, 2 * n:3 * n])
            Z = torch.randn(T, n, generator=g)
            Z[::3, 2::5] = 8.0                            # (a channel that forgets at some tokens only)
            state = torch.randn(6, H, d, d, generator=g)
            Ug, Zg, w0g, ug = U.cuda(), Z.cuda(), w0.cuda(), bonus.cuda()
            rest = (cu.cuda(), seq_slot.cuda(), len(lens), max(lens))
            want_in = R.time_mix_prepare(*cols(U), Z, w0, bonus, H, d)
            got_in = ops.time_mix_prepare(*cols(Ug), Zg, w0g, ug, H, d)
            for x, y in zip(got_in, want_in):
                _near(x, y, 1e-5)
            s_want, s_got = state.clone(), state.cuda()
            want = R.delta_scan(*want_in, s_want, cu, seq_slot, len(lens), max(lens), correct="bonus")
            o = ops.delta_scan(*got_in, s_got, *rest, correct="bonus")
            _near(o, want, 2e-5); _near(s_got, s_want, 2e-5)
            if ops.time_mix_chunks_fits(*cols(Ug), d):
                s_got = state.cuda()
                o = ops.time_mix_chunks(*cols(Ug), Zg, w0g, ug, s_got, *rest, H, d)
                _near(o, want, 2e-5); _near(s_got, s_want, 2e-5)
            if max(lens) == 1:
                s_want, s_got = state.clone(), state.cuda()
                low = slice(3 * n, 3 * n + rank)
                want = R.time_mix_step(*cols(U), U[:, low], w2, w0, bonus, s_want, row_slot, H, d)
                o = ops.time_mix_step(*cols(Ug), Ug[:, low], w2.cuda(), w0g, ug, s_got, row_slot.cuda(), H, d)
                _near(o, want, 2e-5); _near(s_got, s_want, 2e-5)
                _near(ops.tanh_rows(Ug[:, low]), R.tanh_rows(U[:, low]), 1e-5)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_norm_a_head_without_a_weight_against_plain_torch(dtype):
    from inferllm_amd.kernels import ops
    g = torch.Generator().manual_seed(13)
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    for T, width, groups in ((5, 96, 4), (3, 90, 9), (2, 2048, 1), (3, 4096, 32)):
        o, Z = torch.randn(T, width, generator=g) * 2, torch.randn(T, width + 9, generator=g).to(dtype)
        for z in (Z[:, 1:width + 1], Z[:, 8:width + 8]):             # (columns of wider rows)
            want = R.group_norm_gate(o, groups, None, z, 0, "silu", 1e-5, dtype)
            _near(ops.group_norm_gate(o.cuda(), groups, None, Z.cuda()[:, z.storage_offset():z.storage_offset() + width], 0, "silu",
                                      1e-5, dtype), want, tol)


@pytest.mark.parametrize("n_exp, top, groups", [(12, 2, (3, 2)), (64, 6, (8, 3)), (8, 3, (8, 3)), (512, 8, (2, 1)), (9, 2, (3, 1)),
                                                (160, 4, (20, 7)), (7, 3, None)])
def test_choosing_within_groups_against_plain_torch(n_exp, top, groups):
    """Sigmoid scores, corrections that make choice scores negative or turn the choice round, groups whose best pair is
    not the best expert's."""
    from inferllm_amd.kernels import ops
    g = torch.Generator().manual_seed(n_exp)
    for T in (1, 70):
        z, corr = torch.randn(T, n_exp, generator=g) * 2, torch.randn(n_exp, generator=g) * 2 - 1
        idx, wt = R.moe_route(z, corr, top, "sigmoid", 1.0, groups)
        g_idx, g_wt = ops.moe_route(z.cuda(), corr.cuda(), top, "sigmoid", 1.0, groups)
        assert torch.equal(g_idx.cpu(), idx)
        _near(g_wt, wt, 1e-6)
