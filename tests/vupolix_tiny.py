"""Tiny Vupolix configurations and helpers for the tests.  Sizes differ from layer to layer and avoid
equal or trivial values: time mixing with heads times dim above and below the width and ranks of 3 to 9;
attention with 6/2, 5/1, 3/3 and 4/2 heads, rotations of part of a head and of all of it, with and without
scaling, windows of 37, 64 (a page) and 29 tokens and no window; retention with key sizes above and below the
value size, with and without a rotation, decays from 0.3 to 1 (a head that keeps nothing of the past gives a number
times v, of whose size the norm behind it leaves the sign alone); experts in groups of several sizes and in one, one
chosen or several, with and without a shared one; layers without feed-forward; stretches of one and of several
layers that run twice, three times and once, from the first layer on and later; other gains than 1."""
from __future__ import annotations

import os

import torch


def _rot(base, dims, scaling=None):
    """`scaling` = (factor, original, fast, slow)."""
    return {"base": base, "dims": dims, **({"scaling": dict(zip(("factor", "original", "fast", "slow"), scaling))} if scaling else {})}


def _wkv(heads, dim, rank):
    return {"heads": heads, "dim": dim, "rank": rank}


def _left(heads, kv, dim, scale, size=None, rot=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": scale}
    return m | ({"mask": {"size": size}} if size else {}) | ({"rot": rot} if rot else {})


def _right(heads, dim, vdim, decay, rot=None):
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)} | ({"rot": rot} if rot else {})


def _par(left, right):
    return {"left": left, "right": right}


def _moe(ff, experts, top, groups=None, shared=None):
    router = {"experts": experts, "top": top} | ({"groups": dict(zip(("count", "keep"), groups))} if groups else {})
    return {"kind": "moe", "expert": {"ff": ff}, "router": router} | ({"shared": {"ff": shared}} if shared else {})


def _layer(mixer, mlp=None):
    return {"type": "parallel" if "left" in mixer else "wkv", "mixer": mixer, "mlp": mlp}


def _model(layers, vocab, width, eps, gain, logit_scale, loop=None, positions=1024):
    return {"architecture": "Vupolix", "vocab": vocab, "width": width, "max_positions": positions, "norm": {"eps": eps},
            "residual_mult": gain, "logit_scale": logit_scale, "layers": layers,
            **({"loop": dict(zip(("start", "stop", "times"), loop))} if loop else {})}


MIXED = _model([
    _layer(_par(_left(6, 2, 20, 0.4, 37, _rot(5000.0, 8, (3.0, 200, 8.0, 1.5))),
                _right(3, 16, 28, (0.5, 0.93, 0.998), _rot(300.0, 10))), _moe(56, 8, 3, (4, 2), 72)),
    _layer(_wkv(3, 24, 5), _moe(40, 6, 2, (2, 1))),
    _layer(_par(_left(4, 4, 24, 0.25, None, _rot(80.0, 24)), _right(2, 40, 12, (0.97, 0.8), _rot(900.0, 40))), None),
    _layer(_wkv(5, 24, 9), _moe(32, 9, 2, (3, 2), 48)),
], vocab=310, width=96, eps=2e-5, gain=0.6, logit_scale=3.0, loop=(1, 3, 2))

# a width and sizes that are no multiples of 4, a window of exactly one page, no rotations, a decay of exactly 1, one group of all experts, one layer that runs three times, the first and the last layer in the stretch
ODD = _model([
    _layer(_wkv(5, 6, 3), _moe(50, 5, 2, (1, 1))),
    _layer(_par(_left(3, 3, 18, 0.5, 64, _rot(1000.0, 18, (1.5, 60, 6.0, 0.5))), _right(4, 10, 14, (0.3, 1.0, 0.9, 0.99))), None),
    _layer(_par(_left(5, 1, 22, 0.3, 29), _right(1, 26, 6, (0.95,), _rot(40.0, 2))), _moe(30, 6, 1, (6, 3), 44)),
], vocab=131, width=90, eps=3e-6, gain=0.35, logit_scale=0.25, loop=(0, 3, 3))

# every repeat is of one layer; sizes that the matrix cores take
REPEATED = _model([
    _layer(_wkv(2, 32, 16), _moe(64, 4, 2, None, 96)),
    _layer(_par(_left(4, 2, 32, 0.2, 50, _rot(100.0, 16)), _right(2, 32, 64, (0.99, 0.6), _rot(100.0, 32))), _moe(32, 8, 2, (4, 3))),
    _layer(_wkv(4, 64, 32), None),
], vocab=192, width=128, eps=1e-5, gain=0.9, logit_scale=1.5, loop=(2, 3, 2))

# seeds with which bfloat16's rounding stays small through the model: a head's norm magnifies it where the head's
# output nearly cancels (as it may at a sequence's first tokens, where it is a number times v), and a repeated layer
# does so several times
SEEDS = {"MIXED": 12, "ODD": 5, "REPEATED": 5}

CONFIGS = {"MIXED": MIXED, "ODD": ODD, "REPEATED": REPEATED}


def single(mixer, mlp=None, width=64, vocab=200, positions=1024):
    """One layer, for tests of one mechanism and tests that plant a key or a memory."""
    return _model([_layer(mixer, mlp)], vocab=vocab, width=width, eps=1e-6, gain=0.8, logit_scale=2.0, positions=positions)


def write_model(tmp, config: dict, seed: int, dtype=torch.float32, gain: float = 4.0, edit=None) -> str:
    """A random model folder for `config`; every matrix of the layers times `gain` (with the library's small
    random weights a wrong key or a lost state moves nothing), norms, sinks, mixes, bonuses and decays' offsets
    spread, the routers' outputs apart from each other, corrections of both signs and of the scores' size;
    `edit(weights)` may change the float64 weights before they are written."""
    import inferllm_amd as I
    from inferllm_amd.weights.safetensors_io import write_safetensors
    from tiny import read_weights
    d = os.path.join(str(tmp), f"vupolix_{seed}_{abs(hash(repr(config))) % 10**8}_{str(dtype)[6:]}")
    I.write_random_model(d, I.config_from_dict(config), seed=seed, dtype=torch.float32)
    w = {}
    g = torch.Generator().manual_seed(seed)
    rnd = lambda shape: torch.randn(shape, generator=g, dtype=torch.float64)
    for n, t in read_weights(d).items():
        t = t.double()
        if n.endswith(".w0"):
            t = rnd(t.shape) * 2.0 - 1.5                  # channels that forget at different speeds, some at once
        elif n.endswith(".mix.u"):
            t = rnd(t.shape)
        elif ".mu." in n:
            t = 0.5 + rnd(t.shape) * 0.5                  # (also beyond 0 and 1)
        elif n.endswith(".sink"):
            t = rnd(t.shape) * 2.0
        elif n.endswith(".correction"):
            # choice scores of both signs; in bfloat16 so far apart that the rounding of the activations turns
            # hardly a choice
            t = rnd(t.shape) * (0.7 if dtype == torch.float32 else 4.0) - 0.5
        elif n.endswith(".router"):
            t = rnd(t.shape) * (2.0 / t.shape[1] ** 0.5)
        elif n.endswith(".w1") or n.endswith(".w2"):
            t = t * 20
        elif "norm" in n or n.endswith(".out"):
            t = 1.0 + rnd(t.shape) * 0.3
        elif n == "embed":
            t = t * 40
        elif t.dim() == 2:
            t = t * gain
        w[n] = t
    if edit is not None:
        edit(w)
    write_safetensors(os.path.join(d, "model.safetensors"), [(n, t.to(dtype)) for n, t in w.items()],
                      metadata={"format": "pt"})
    return d


def weights64(model_dir: str):
    from tiny import read_weights
    return {n: t.double() for n, t in read_weights(model_dir).items()}


def _mark(w, token: int, column: int, size: float = 6.0) -> None:
    """Give `token` alone a large entry in `column` of the embedded rows."""
    w["embed"][:, column] = 0.0
    w["embed"][token, column] = size


def plant_key(w, config: dict, key_token: int, query_token: int) -> None:
    """Change layer 0's attention so that `query_token`'s score for `key_token` stands far above every other
    score, in every head: each of the two tokens alone has a large entry in a column of its own, the last query
    dim of every head, which is not rotated, reads the query token's column and the same dim of every key head
    the key token's column alone, and the key token's keys, which are its values, are large.  The other mixer's
    output is held small.  Both tokens must occur nowhere else in the sequence."""
    m, p = config["layers"][0]["mixer"]["left"], "l0.mix.left."
    _mark(w, key_token, 0)
    _mark(w, query_token, 1)
    last = m["dim"] - 1
    w[p + "k"][:, 0] += 1.0
    for n, heads, column in (("q", m["heads"], 1), ("k", m["kv_heads"], 0)):
        for hh in range(heads):
            at = hh * m["dim"] + last
            w[p + n][at, :] = 0.0
            w[p + n][at, column] = 5.0
    w["l0.mix.right.out"][:] *= 0.1


def plant_memory(w, config: dict, token: int) -> None:
    """Change layer 0's recurrent mixer so that `token` is written into the state with a weight far above
    every other token's and is hardly forgotten afterwards (retention's decays are the configuration's)."""
    _mark(w, token, 0)
    if config["layers"][0]["type"] == "wkv":
        w["l0.mix.k"][:, 0] += 4.0
        w["l0.mix.v"][:, 0] += 4.0
        w["l0.mix.w0"][:] = -11.0
        w["l0.mix.w2"][:] = 0.0
    else:
        w["l0.mix.right.k"][:, 0] += 4.0
        w["l0.mix.right.v"][:, 0] += 4.0
        w["l0.mix.left.out"][:] *= 0.1
