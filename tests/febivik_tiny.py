"""Tiny Febivik configurations and helpers for the tests.  Sizes differ from layer to layer and avoid
equal or trivial values: attention with 6/2, 4/4, 3/1 and 10/5 heads, key sizes above and below the
value size, rotations of part of a head and of all of it, with and without scaling; windows of 37,
64 (a page) and 29 tokens that keep 3, 1, 70 (more than a page) and no first tokens, and no window;
lightning attention with key sizes above and below the value size, decays from 0 to 1; the delta rule
with ranks of 3 to 9; dense feed-forwards, experts with and without a shared one, one chosen or
several, layers without feed-forward; every order of the three kinds of layer."""
from __future__ import annotations

import os

import torch

import plain_febivik as P


def _rot(base, dims, factor=None):
    return {"base": base, "dims": dims, **({"scaling": {"factor": factor}} if factor else {})}


def _att(heads, kv, dim, vdim, scale, rot=None, size=None, keep=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale}
    if rot is not None:
        m["rot"] = rot
    if size is not None:
        m["mask"] = {"size": size, **({"keep_first": keep} if keep is not None else {})}
    return m


def _light(heads, dim, vdim, decay):
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}


def _delta(heads, dim, rank):
    return {"heads": heads, "dim": dim, "rank": rank}


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(ff, experts, top, scale=None, shared=None):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, **({"scale": scale} if scale else {})},
            **({"shared": {"ff": shared}} if shared else {})}


def _layer(kind, mixer, mlp=None):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def _model(layers, vocab, width, eps, positions):
    return {"architecture": "Febivik", "vocab": vocab, "width": width, "max_positions": positions,
            "norm": {"eps": eps}, "layers": layers}


MIXED = _model([
    _layer("attention", _att(6, 2, 20, 12, 0.4, _rot(5000.0, 8, 3.0), 37, 3), _moe(56, 5, 2, 1.7, 72)),
    _layer("lightning", _light(3, 16, 28, (0.5, 0.93, 0.998)), _dense(112)),
    _layer("general_delta", _delta(2, 24, 5), _moe(40, 6, 3, 0.6)),
    _layer("attention", _att(4, 4, 24, 32, 0.25, _rot(300.0, 24)), None),
    _layer("lightning", _light(2, 40, 12, (0.97, 0.8)), _moe(32, 4, 1, 2.5, 48)),
    _layer("general_delta", _delta(3, 12, 9), _dense(64)),
], vocab=310, width=96, eps=2e-5, positions=1024)

# a width that is no multiple of 4, sizes that are no multiple of 4, a window of exactly one page, more
# kept tokens than a page holds, decays of exactly 0 and 1, a delta layer first
ODD = _model([
    _layer("general_delta", _delta(5, 6, 3), _dense(50)),
    _layer("attention", _att(3, 1, 18, 22, 0.5, _rot(1000.0, 18, 1.5), 64, 1), None),
    _layer("lightning", _light(4, 10, 14, (0.0, 1.0, 0.9, 0.99)), _moe(30, 7, 2, None, 44)),
    _layer("attention", _att(10, 5, 8, 16, 0.3, _rot(40.0, 2), 29, 70), _moe(22, 3, 3, 0.9)),
], vocab=131, width=90, eps=3e-6, positions=1024)

# nothing is kept per token
NO_KEYS = _model([
    _layer("lightning", _light(2, 16, 8, (0.99, 0.6)), _dense(48)),
    _layer("general_delta", _delta(4, 16, 7), None),
], vocab=120, width=48, eps=1e-5, positions=400)

CONFIGS = {"MIXED": MIXED, "ODD": ODD, "NO_KEYS": NO_KEYS}


def single(kind, mixer, mlp=None, width=64, vocab=200, positions=1024):
    """One layer, for tests of one mechanism and tests that plant a key or a memory."""
    return _model([_layer(kind, mixer, mlp)], vocab=vocab, width=width, eps=1e-6, positions=positions)


def write_model(tmp, config: dict, seed: int, dtype=torch.float32, gain: float = 4.0, edit=None) -> str:
    """A random model folder for `config`; every matrix of the layers times `gain` (with the library's
    small random weights a wrong key or a lost state moves nothing), biases, norms and the decays'
    offsets spread, the routers' outputs apart from each other, the embedded rows of about unit size;
    `edit(weights)` may change the float64 weights before they are written."""
    import inferllm_amd as I
    from inferllm_amd.weights.safetensors_io import write_safetensors
    from tiny import read_weights
    d = os.path.join(str(tmp), f"febivik_{seed}_{abs(hash(repr(config))) % 10**8}_{str(dtype)[6:]}")
    I.write_random_model(d, I.config_from_dict(config), seed=seed, dtype=torch.float32)
    w = {}
    g = torch.Generator().manual_seed(seed)
    rnd = lambda shape: torch.randn(shape, generator=g, dtype=torch.float64)
    for n, t in read_weights(d).items():
        t = t.double()
        if n.endswith(".w0"):
            t = rnd(t.shape) * 2.0 - 2.0                  # channels that forget at different speeds
        elif n.endswith(".a.b"):
            t = rnd(t.shape) * 2.0
        elif n.endswith(".act"):
            t = rnd(t.shape)
        elif n.endswith(".b"):
            t = rnd(t.shape) * 0.3
        elif n.endswith(".router"):
            t = rnd(t.shape) * (2.0 / t.shape[1] ** 0.5)
        elif n.endswith(".w1") or n.endswith(".w2"):
            t = t * 20
        elif "norm" in n:
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
    """Change layer 0's attention so that `query_token`'s score for `key_token` stands far above every
    other score, in every head: each of the two tokens alone has a large entry in a column of its own,
    the last query dim of every head, which is not rotated, reads the query token's column and the
    same dim of every key head the key token's column alone, and the key token's values are large.
    (The norm a head leaves the query close to its last dim, and every other key without one.)
    Both tokens must occur nowhere else in the sequence."""
    m, p = config["layers"][0]["mixer"], "l0.mix."
    _mark(w, key_token, 0)
    _mark(w, query_token, 1)
    last = m["dim"] - 1
    for n, heads, column in (("q", m["heads"], 1), ("k", m["kv_heads"], 0)):
        for hh in range(heads):
            at = hh * m["dim"] + last
            w[p + n][at, :] = 0.0
            w[p + n][at, column] = 8.0
            w[p + n + ".b"][at] = 0.0
        w[p + n + ".norm"][last] = 1.0
    w[p + "v"][:, 0] += 2.0


def plant_memory(w, config: dict, token: int) -> None:
    """Change layer 0's recurrent mixer so that `token` is written into the state with a weight far
    above every other token's and is hardly forgotten or removed afterwards (lightning attention's
    decays are the configuration's)."""
    _mark(w, token, 0)
    w["l0.mix.k"][:, 0] += 4.0
    w["l0.mix.v"][:, 0] += 4.0
    if config["layers"][0]["type"] == "general_delta":
        w["l0.mix.w0"][:] = -7.0
        w["l0.mix.w2"][:] = 0.0
        w["l0.mix.a"][:] = 0.0
        w["l0.mix.a.b"][:] = -9.0


def rel_err(got: torch.Tensor, want: torch.Tensor) -> float:
    return float((got.double().cpu() - want).abs().max() / want.abs().max())
