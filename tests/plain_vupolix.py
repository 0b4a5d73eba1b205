"""Vupolix, plainly: one function per mechanism, float64 on the CPU, token by token where the
design is recurrent.  It shares no code with the library; the tests compare the engine with it.

Notation: h holds a sublayer's input rows [T, E]; a matrix W [out, in] acts on a row as W h, which
for all rows at once is h @ W.T.  Positions count from 0.
"""
from __future__ import annotations

import math

import torch


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(x):
    return x * torch.sigmoid(x)


# ---------------------------------------------------------------- recurrent time mixing
def token_before(h):
    """Every token's predecessor; zeros for the first token."""
    return torch.cat([torch.zeros_like(h[:1]), h[:-1]])


def wkv(h, w, p, m, eps):
    """o_t = (S + diag(u) k v^T)^T r with the state S before the token, then S <- diag(w) S + k v^T."""
    H, d = m["heads"], m["dim"]
    T = h.shape[0]
    step = token_before(h) - h
    mix = lambda n: h + step * w[p + "mu." + n]
    r, k, v = ((mix(n) @ w[p + n].T).view(T, H, d) for n in ("r", "k", "v"))
    gate = silu(mix("g") @ w[p + "g"].T)
    low = torch.tanh(mix("w") @ w[p + "w1"].T) @ w[p + "w2"].T
    decay = torch.exp(-torch.exp(low + w[p + "w0"])).view(T, H, d)
    u = w[p + "u"]
    S = torch.zeros(H, d, d, dtype=h.dtype)
    o = torch.zeros(T, H, d, dtype=h.dtype)
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        o[t] = ((S + u[:, :, None] * kv) * r[t][:, :, None]).sum(1)
        S = decay[t][:, :, None] * S + kv
    y = unit_rms(o, eps).reshape(T, H * d) * w[p + "norm"]
    return (y * gate) @ w[p + "o"].T


# ---------------------------------------------------------------- windowed attention
def frequencies(rot):
    """(frequencies [dims / 2], gain of cos and sin)."""
    dims, base = rot["dims"], rot["base"]
    i = torch.arange(dims // 2, dtype=torch.float64)
    f = torch.tensor(float(base), dtype=torch.float64) ** (-2.0 * i / dims)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    at = lambda turns: dims * math.log(sc["original"] / (turns * 2 * math.pi)) / (2 * math.log(base))
    lo, hi = max(math.floor(at(sc["fast"])), 0), min(math.ceil(at(sc["slow"])), dims - 1)
    share = torch.clamp((i - lo) / max(hi - lo, 0.001), 0, 1)
    return (1 - share) * f + share * f / sc["factor"], 1.0 + 0.1 * math.log(sc["factor"])


def rotate(x, rot):
    """x [T, heads, d]: the first rot.dims of every head turned by position, i with i + dims / 2."""
    if not rot:
        return x
    f, gain = frequencies(rot)
    dims, half = rot["dims"], rot["dims"] // 2
    a = torch.arange(x.shape[0], dtype=torch.float64)[:, None] * f[None, :]
    c, s = (gain * torch.cos(a))[:, None, :].to(x.dtype), (gain * torch.sin(a))[:, None, :].to(x.dtype)
    out = x.clone()
    first, second = x[..., :half], x[..., half:dims]
    out[..., :half], out[..., half:dims] = first * c - second * s, second * c + first * s
    return out


def visible_keys(T, mask, edge_shift=0):
    """[T, T] bool: i sees j <= i within the window.  `edge_shift` moves the window's far edge: what
    an implementation that is off by one there would compute."""
    back = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    seen = back >= 0
    return seen & (back < mask["size"] + edge_shift) if mask else seen


def attention(h, w, p, m, edge_shift=0, sink_on=True):
    """The values are the unrotated keys; a sink in the softmax's denominator; one gate a head."""
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    T = h.shape[0]
    q, k = (h @ w[p + "q"].T).view(T, H, d), (h @ w[p + "k"].T).view(T, G, d)
    v = k
    q, k = rotate(q, m.get("rot")), rotate(k, m.get("rot"))
    seen = visible_keys(T, m.get("mask"), edge_shift)
    gate = torch.sigmoid(h @ w[p + "g"].T)
    out = torch.zeros(T, H, d, dtype=h.dtype)
    for hh in range(H):
        g = hh // (H // G)
        s = (q[:, hh] @ k[:, g].T * m["scale"]).masked_fill(~seen, float("-inf"))
        if sink_on:
            s = torch.cat([s, w[p + "sink"][hh].expand(T, 1)], 1)
        e = torch.exp(s - s.max(1, keepdim=True).values)
        e = e / e.sum(1, keepdim=True)
        out[:, hh] = (e[:, :T] @ v[:, g]) * gate[:, hh:hh + 1]
    return out.reshape(T, H * d) @ w[p + "o"].T


# ---------------------------------------------------------------- retention
def retention(h, w, p, m, eps):
    """S <- decay_h S + k v^T, o = S^T q, with q and k rotated and k times dim^(-1/2)."""
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q, k = rotate((h @ w[p + "q"].T).view(T, H, dk), m.get("rot")), rotate((h @ w[p + "k"].T).view(T, H, dk), m.get("rot"))
    k = k / math.sqrt(dk)
    v = (h @ w[p + "v"].T).view(T, H, dv)
    g = torch.tensor(m["decay"], dtype=h.dtype)[:, None, None]
    S = torch.zeros(H, dk, dv, dtype=h.dtype)
    o = torch.zeros(T, H, dv, dtype=h.dtype)
    for t in range(T):
        S = g * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    return (unit_rms(o, eps).reshape(T, H * dv) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel(h, w, p, m, eps, edge_shift=0, sink_on=True):
    a = attention(h, w, p + "left.", m["left"], edge_shift, sink_on)
    b = retention(h, w, p + "right.", m["right"], eps)
    return (unit_rms(a, eps) * w[p + "left.out"] + unit_rms(b, eps) * w[p + "right.out"]) / 2


# ---------------------------------------------------------------- experts
def gated_expert(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def choose(score, choice, top, groups):
    """Indices of the `top` largest choice scores within the best groups of neighbours."""
    allowed = torch.full_like(choice, float("-inf"))
    if groups:
        size = choice.numel() // groups["count"]
        of_group = []
        for j in range(groups["count"]):
            best = sorted(choice[j * size:(j + 1) * size].tolist(), reverse=True)
            of_group.append(sum(best[:2]))
        keep = sorted(range(groups["count"]), key=lambda j: -of_group[j])[:groups["keep"]]
        for j in keep:
            allowed[j * size:(j + 1) * size] = choice[j * size:(j + 1) * size]
    else:
        allowed = choice
    return torch.topk(allowed, top).indices.tolist()


def experts(h, w, p, mlp):
    """The chosen experts' outputs weighted by their sigmoid scores (not renormalized), and the
    shared expert's."""
    r = mlp["router"]
    s = torch.sigmoid(h @ w[p + "router"].T)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e in choose(s[t], s[t] + w[p + "correction"], r["top"], r.get("groups")):
            out[t] += s[t, e] * gated_expert(h[t:t + 1], w, f"{p}e{e}.")[0]
    if mlp.get("shared"):
        out = out + gated_expert(h, w, p + "shared.")
    return out


# ---------------------------------------------------------------- the model
def order_of_layers(config):
    """[(layer, whether the embedding output is added first)] of one token's way."""
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    out = [(i, False) for i in range(a)]
    for turn in range(loop["times"]):
        out += [(i, turn > 0 and i == a) for i in range(a, b)]
    return out + [(i, False) for i in range(b, n)]


def forward(config, w, ids, layers_out=None, edge_shift=0, sink_on=True):
    """float64 logits [T, vocab] of one sequence from its first token on."""
    eps, gain = config["norm"]["eps"], config["residual_mult"]
    norm = lambda x, n: unit_rms(x, eps) * w[n]
    first = norm(w["embed"][torch.as_tensor(ids, dtype=torch.long)], "embed.norm")
    x = first
    for i, again in order_of_layers(config):
        layer, L, p = config["layers"][i], f"l{i}.", f"l{i}.mix."
        if again:
            x = x + first
        h = norm(x, L + "norm1")
        y = (wkv(h, w, p, layer["mixer"], eps) if layer["type"] == "wkv"
             else parallel(h, w, p, layer["mixer"], eps, edge_shift, sink_on))
        x = x + gain * norm(y, L + "norm1b")
        if layer.get("mlp") is not None:
            x = x + gain * norm(experts(norm(x, L + "norm2"), w, L + "mlp.", layer["mlp"]), L + "norm2b")
        if layers_out is not None:
            layers_out.append(x.clone())
    return norm(x, "final.norm") @ w["head"].T * config["logit_scale"]


def generate_greedy(config, w, prompt, n_new):
    ids, out = list(prompt), []
    for _ in range(n_new):
        t = int(torch.argmax(forward(config, w, ids)[-1]))
        ids.append(t)
        out.append(t)
    return out
