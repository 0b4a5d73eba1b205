"""Febivik, plainly: one function per mechanism, float64 on the CPU, token by token where the
design is recurrent.  It shares no code with the library; the tests compare the engine with it.

Notation: h holds a sublayer's input rows [T, E]; a matrix W [out, in] acts on a row as W h, which
for all rows at once is h @ W.T.  Positions count from 0.
"""
from __future__ import annotations

import math

import torch


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, w, b, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w + b


def silu(x):
    return x * torch.sigmoid(x)


def softplus(x):
    return torch.where(x > 30, x, torch.log1p(torch.exp(torch.clamp(x, max=30))))


def xielu(z, p, q):
    """z > 0: softplus(p) z^2 + z / 2;  z <= 0: (1/2 + softplus(q)) (e^z - 1 - z) + z / 2."""
    neg = torch.clamp(z, max=0)
    below = (0.5 + softplus(q)) * (torch.expm1(neg) - neg)
    return torch.where(z > 0, softplus(p) * z * z, below) + 0.5 * z


def rotate(x, base, dims, factor, first_pos=0):
    """x [T, heads, d]: the first `dims` of every head turned by position, i with i + dims / 2, every
    frequency divided by `factor`."""
    T, half = x.shape[0], dims // 2
    f = torch.tensor(base, dtype=torch.float64) ** (-2.0 * torch.arange(half, dtype=torch.float64) / dims) / factor
    a = (torch.arange(T, dtype=torch.float64) + first_pos)[:, None] * f[None, :]
    c, s = torch.cos(a)[:, None, :].to(x.dtype), torch.sin(a)[:, None, :].to(x.dtype)
    out = x.clone()
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half], out[..., half:dims] = u * c - v * s, v * c + u * s
    return out


def visible_keys(T, mask, edge_shift=0, keep_shift=0):
    """[T, T] bool: i sees j <= i within the window, or among the kept first tokens.  The shifts move
    the window's far edge and the number of kept tokens: what an implementation that is off by one
    there would compute."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    if mask:
        seen = seen & ((i - j < mask["size"] + edge_shift) | (j < mask.get("keep_first", 0) + keep_shift))
    return seen


def attention(h, w, p, m, eps, edge_shift=0, keep_shift=0):
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = (h @ w[p + "q"].T + w[p + "q.b"]).view(T, H, dk)
    k = (h @ w[p + "k"].T + w[p + "k.b"]).view(T, G, dk)
    v = (h @ w[p + "v"].T + w[p + "v.b"]).view(T, G, dv)
    q, k = unit_rms(q, eps) * w[p + "q.norm"], unit_rms(k, eps) * w[p + "k.norm"]
    rot = m.get("rot")
    if rot:
        factor = (rot.get("scaling") or {}).get("factor", 1.0)
        q, k = rotate(q, rot["base"], rot["dims"], factor), rotate(k, rot["base"], rot["dims"], factor)
    seen = visible_keys(T, m.get("mask"), edge_shift, keep_shift)
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for hh in range(H):
        g = hh // (H // G)
        s = (q[:, hh] @ k[:, g].T * m["scale"]).masked_fill(~seen, float("-inf"))
        out[:, hh] = torch.softmax(s, 1) @ v[:, g]
    return out.reshape(T, H * dv) @ w[p + "o"].T


def lightning(h, w, p, m, eps):
    """S <- decay_h S + k v^T, o = S^T q, with q, k and v through SiLU; one norm over all heads."""
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = silu(h @ w[p + "q"].T).view(T, H, dk)
    k = silu(h @ w[p + "k"].T).view(T, H, dk)
    v = silu(h @ w[p + "v"].T).view(T, H, dv)
    g = torch.tensor(m["decay"], dtype=h.dtype)[:, None, None]
    S = torch.zeros(H, dk, dv, dtype=h.dtype)
    o = torch.zeros(T, H, dv, dtype=h.dtype)
    for t in range(T):
        S = g * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    y = unit_rms(o.reshape(T, H * dv), eps) * w[p + "norm"]
    return (y * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def general_delta(h, w, p, m, eps):
    """S_new = diag(w) S - (a u) (u^T S) + k v^T with the unit key u; o = S_new^T r."""
    H, d = m["heads"], m["dim"]
    T = h.shape[0]
    heads = lambda n: (h @ w[p + n].T).view(T, H, d)
    r, k, v = heads("r"), heads("k"), heads("v")
    low = torch.tanh(h @ w[p + "w1"].T) @ w[p + "w2"].T
    decay = torch.exp(-math.exp(-0.5) * torch.sigmoid(low + w[p + "w0"])).view(T, H, d)
    a = torch.sigmoid(h @ w[p + "a"].T + w[p + "a.b"]).view(T, H, d)
    u = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
    S = torch.zeros(H, d, d, dtype=h.dtype)
    o = torch.zeros(T, H, d, dtype=h.dtype)
    for t in range(T):
        read = (S * u[t][:, :, None]).sum(1)                     # u^T S per head
        S = (decay[t][:, :, None] * S - (a[t] * u[t])[:, :, None] * read[:, None, :]
             + k[t][:, :, None] * v[t][:, None, :])
        o[t] = (S * r[t][:, :, None]).sum(1)
    y = unit_rms(o, eps).reshape(T, H * d) * w[p + "norm"]
    return (y * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def dense(h, w, p):
    act = w[p + "act"]
    return xielu(h @ w[p + "up"].T, act[0], act[1]) @ w[p + "down"].T


def squared_relu_expert(h, w, p):
    return torch.clamp(h @ w[p + "up"].T, min=0) ** 2 @ w[p + "down"].T


def experts(h, w, p, mlp):
    """The chosen experts' outputs weighted by their softmax scores times the router's scale (not
    renormalized), and the shared expert's."""
    r = mlp["router"]
    s = torch.softmax(h @ w[p + "router"].T, -1)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e in torch.topk(s[t], r["top"]).indices.tolist():
            out[t] += s[t, e] * r.get("scale", 1.0) * squared_relu_expert(h[t:t + 1], w, f"{p}e{e}.")[0]
    if mlp.get("shared"):
        out = out + squared_relu_expert(h, w, p + "shared.")
    return out


def forward(config, w, ids, layers_out=None, edge_shift=0, keep_shift=0):
    """float64 logits [T, vocab] of one sequence from its first token on."""
    eps = config["norm"]["eps"]
    norm = lambda x, n: layer_norm(x, w[n], w[n + ".b"], eps)
    x = w["embed"][torch.as_tensor(ids, dtype=torch.long)]
    for i, layer in enumerate(config["layers"]):
        L, p, m = f"l{i}.", f"l{i}.mix.", layer["mixer"]
        if layer["type"] == "attention":
            y = attention(x, w, p, m, eps, edge_shift, keep_shift)
        else:
            y = {"lightning": lightning, "general_delta": general_delta}[layer["type"]](x, w, p, m, eps)
        x = x + norm(y, L + "norm1")
        mlp = layer.get("mlp")
        if mlp is not None:
            y = dense(x, w, L + "mlp.") if mlp["kind"] == "dense" else experts(x, w, L + "mlp.", mlp)
            x = x + norm(y, L + "norm2")
        if layers_out is not None:
            layers_out.append(x.clone())
    return norm(x, "final.norm") @ w["head"].T


def generate_greedy(config, w, prompt, n_new):
    ids, out = list(prompt), []
    for _ in range(n_new):
        t = int(torch.argmax(forward(config, w, ids)[-1]))
        ids.append(t)
        out.append(t)
    return out
