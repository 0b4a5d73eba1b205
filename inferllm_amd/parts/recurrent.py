"""Mixers that keep a matrix of state per head and update it by the plain gated rule
S <- g S + k (w v)^T, o = S^T q: a state-space mixer with a scalar decay a head, and a matrix
memory with exponential gates; gated linear attention, which is that rule with a decay per key
channel; lightning attention and retention, with one fixed decay a head; the delta rule with a removal
vector of its own; time mixing with a token shift and a bonus for the current token; and a gated linear
recurrent unit, whose state is one number a channel."""
from __future__ import annotations

import math
from typing import Dict, Sequence

import torch

from ..cache.manager import StateSpec
from ..kernels import ops
from ..weights.loader import TensorWant
from .attention import _fuse
from .base import Mixer, StepContext, register_part


@register_part("mixer", "state_space_duality")
class StateSpaceDuality(Mixer):
    """A selective state-space mixer with one decay a head.  The input projection gives, side by
    side, [z: H dv | x: H dv | B: G N | C: G N | dt: H].  x, B and C pass a short causal
    convolution per channel (`conv` taps with a bias, the last tap on the token itself, zeros ahead
    of the sequence) and SiLU.  With step = softplus(dt + dt_bias), per head h of group
    h / (H / G):

        S <- exp(-exp(A_log[h]) step) S + step B x^T      (S is N x dv)
        y = S^T C + D[h] x

    y (heads side by side) times silu(z), then an RMS norm in `norm_groups` equal parts of the row
    (each by its own root mean square, `eps`), times `norm`, then the output projection.

    Kept per sequence: S (float32) and the convolution's last conv - 1 inputs.  A step goes on from
    whatever the slot holds, by one token or by many.  Everything that enters the recurrence is
    float32; the projections take the engine's dtype.
    """

    graph_safe_prompts = True
    takes_continuations = True

    def __init__(self, hidden_size: int, num_heads: int, groups: int, state_size: int, value_dim: int,
                 conv: int, norm_groups: int, eps: float, tensors=None):
        super().__init__(tensors)
        if num_heads % groups:
            raise ValueError(f"{num_heads} heads are not a multiple of {groups} groups")
        if not 1 <= int(conv) <= 8:
            raise ValueError(f"state-space mixer: {conv} taps; the kernels take 1 to 8")
        if state_size > 256:
            raise ValueError(f"state-space mixer: a state of {state_size} rows is beyond the kernels' limit of 256")
        if (num_heads * value_dim) % norm_groups:
            raise ValueError(f"{num_heads * value_dim} columns do not split into {norm_groups} equal parts")
        self.E, self.H, self.G = int(hidden_size), int(num_heads), int(groups)
        self.N, self.dv, self.taps = int(state_size), int(value_dim), int(conv)
        self.norm_groups, self.eps = int(norm_groups), float(eps)
        self.inner = self.H * self.dv
        self.C = self.inner + 2 * self.G * self.N                # channels of the convolution

    def shapes(self) -> Dict[str, TensorWant]:
        keep = dict(keep_stored=True)
        return {"in": TensorWant((2 * self.inner + 2 * self.G * self.N + self.H, self.E)),
                "conv": TensorWant((self.C, self.taps), **keep), "conv_bias": TensorWant((self.C,), **keep),
                "dt_bias": TensorWant((self.H,), **keep), "A_log": TensorWant((self.H,), **keep),
                "D": TensorWant((self.H,), init="ones_normal", **keep),
                "norm": TensorWant((self.inner,), init="ones_normal", **keep),
                "o": TensorWant((self.E, self.inner))}

    def state_spec(self):
        return {"S": StateSpec((self.H, self.N, self.dv), torch.float32),
                "tail": StateSpec((max(self.taps - 1, 1), self.C), None)}

    def load(self, tensors) -> None:
        take = lambda n: self._take(tensors, n)
        f32 = lambda n: take(n).to(torch.float32).contiguous()
        self.w_in = ops.decode_weight(take("in").contiguous(), "plain", self.decode_copies)
        self.w_o = ops.decode_weight(take("o").contiguous(), "plain", self.decode_copies)
        self.conv_w, self.conv_b = f32("conv"), f32("conv_bias")
        self.dt_bias, self.a_log, self.D = f32("dt_bias"), f32("A_log"), f32("D")
        self.norm_w = take("norm").contiguous()

    def tunables(self):
        return (("plain", self.w_o, {}),)

    def forward(self, h, ctx: StepContext, line, writes_cache, position):
        U = ops.linear(h, self.w_in)
        state = ctx.cache.state_line(line)
        S, tail = state["S"], state["tail"]
        qn, kn, vv, step, dec = ops.ssm_prepare(
            U, self.inner, 2 * self.inner + 2 * self.G * self.N, self.conv_w, self.conv_b, tail,
            ctx.row_slot, self.a_log, self.dt_bias, self.G, self.H, self.N, self.dv,
            update_tail=not ctx.prefill)
        if ctx.prefill:
            ops.delta_conv_tail(U, tail, ctx.cu_seqlens, ctx.seq_slot, ctx.n_seqs, self.taps,
                                col_off=self.inner)
        o = ops.delta_scan(qn, kn, vv, step, dec, S, ctx.cu_seqlens, ctx.seq_slot, ctx.n_seqs,
                           ctx.max_rows if ctx.prefill else 1, correct=False)
        y = ops.ssm_finish(o, vv, self.D, U, 0, self.norm_w, self.norm_groups, self.eps, ctx.act_dtype)
        return ops.linear(y, self.w_o)


@register_part("mixer", "matrix_memory")
class MatrixMemory(Mixer):
    """A matrix memory with exponential gates (the mLSTM cell).  q = W_q h dk^-1/2, k = W_k h, v = W_v h
    per head; per head a log input gate i = cap tanh((W_i h + b_i) / cap) and a log forget gate
    f = logsigmoid(cap tanh((W_f h + b_f) / cap)).  With a running maximum m that starts at 0:

        m_t = max(f + m_(t-1), i)
        S <- exp(f + m_(t-1) - m_t) S + exp(i - m_t) k v^T,   n likewise with k alone
        o = S^T q / (max(|n . q|, exp(-m_t)) + 1e-6)

    Each head's o is divided by its root mean square (`eps`); the heads side by side times `norm`
    (all heads' width), times sigmoid(W_g h), then the output projection.

    Kept per sequence, float32: S with n as one more column ([H, dk, dv + 1]) and m [H].  A step
    goes on from whatever the slot holds.  Gates, maxima, decays and the state are float32; the
    projections take the engine's dtype.
    """

    graph_safe_prompts = True
    takes_continuations = True

    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, value_dim: int, gate_cap: float,
                 eps: float, tensors=None):
        super().__init__(tensors)
        if key_dim > 256:
            raise ValueError(f"matrix memory: a key size of {key_dim} is beyond the kernels' limit of 256")
        if not float(gate_cap) > 0:
            raise ValueError(f"matrix memory: the gates' cap must be positive, got {gate_cap!r}")
        self.E, self.H, self.dk, self.dv = int(hidden_size), int(num_heads), int(key_dim), int(value_dim)
        self.cap, self.eps = float(gate_cap), float(eps)

    def shapes(self) -> Dict[str, TensorWant]:
        E, H, dk, dv = self.E, self.H, self.dk, self.dv
        keep = dict(keep_stored=True)
        return {"q": TensorWant((H * dk, E)), "k": TensorWant((H * dk, E)), "v": TensorWant((H * dv, E)),
                "g": TensorWant((H * dv, E)), "i": TensorWant((H, E)), "f": TensorWant((H, E)),
                "i_bias": TensorWant((H,), **keep), "f_bias": TensorWant((H,), **keep),
                "norm": TensorWant((H * dv,), init="ones_normal", **keep), "o": TensorWant((E, H * dv))}

    def state_spec(self):
        return {"S": StateSpec((self.H, self.dk, self.dv + 1), torch.float32),
                "m": StateSpec((self.H,), torch.float32)}

    def load(self, tensors) -> None:
        take = lambda n: self._take(tensors, n)
        H, dk, dv = self.H, self.dk, self.dv
        # one product for everything that reads h: [q | k | v | i | f | g]
        self.w_in = ops.decode_weight(_fuse([take(n) for n in ("q", "k", "v", "i", "f", "g")]), "plain",
                                      self.decode_copies)
        self.i_off = 2 * H * dk + H * dv
        self.f_off, self.z_off = self.i_off + H, self.i_off + 2 * H
        self.i_bias = take("i_bias").to(torch.float32).contiguous()
        self.f_bias = take("f_bias").to(torch.float32).contiguous()
        self.norm_w = take("norm").contiguous()
        self.w_o = ops.decode_weight(take("o").contiguous(), "plain", self.decode_copies)

    def tunables(self):
        return (("plain", self.w_o, {}),)

    def forward(self, h, ctx: StepContext, line, writes_cache, position):
        U = ops.linear(h, self.w_in)
        state = ctx.cache.state_line(line)
        qn, kn, vv, weight, dec, em = ops.memory_prepare(
            U, self.i_off, self.f_off, self.i_bias, self.f_bias, self.cap, state["m"], ctx.cu_seqlens,
            ctx.seq_slot, ctx.n_seqs, self.H, self.dk, self.dv)
        o = ops.delta_scan(qn, kn, vv, weight, dec, state["S"], ctx.cu_seqlens, ctx.seq_slot, ctx.n_seqs,
                           ctx.max_rows if ctx.prefill else 1, correct=False)
        y = ops.memory_finish(o, em, self.norm_w, U, self.z_off, self.eps, ctx.act_dtype)
        return ops.linear(y, self.w_o)


@register_part("mixer", "gated_linear_attention")
class GatedLinearAttention(Mixer):
    """Per head a matrix of state S [key_dim, value_dim] with a decay per key channel:

        q = W_q h key_dim^-1/2,  k = W_k h,  v = W_v h
        alpha = sigmoid(W_a2 (W_a1 h) + b)^(1 / tau)             one a head and key channel
        S <- diag(alpha) S + k v^T;   o = S^T q
        out = W_o (o / rms(o) * norm * silu(W_g h))

    rms over a head's value dims with `eps`; `norm` [value_dim] is shared by the heads.  Kept per
    sequence: S (float32).  A step goes on from whatever the slot holds.  Decays, their logarithms
    and the state are float32; the projections take the engine's dtype.
    """

    graph_safe_prompts = True
    takes_continuations = True

    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, value_dim: int, decay_rank: int,
                 tau: float, eps: float, tensors=None):
        super().__init__(tensors)
        if key_dim > 256 or value_dim > 256:
            raise ValueError(f"gated linear attention: head sizes {key_dim}, {value_dim} are beyond the kernels' limit of 256")
        if not float(tau) > 0 or int(decay_rank) <= 0:
            raise ValueError("gated linear attention: tau and the decays' rank must be positive")
        self.E, self.H, self.dk, self.dv = int(hidden_size), int(num_heads), int(key_dim), int(value_dim)
        self.ra, self.tau, self.eps = int(decay_rank), float(tau), float(eps)

    def shapes(self) -> Dict[str, TensorWant]:
        E, H, dk, dv = self.E, self.H, self.dk, self.dv
        keep = dict(keep_stored=True)
        return {"q": TensorWant((H * dk, E)), "k": TensorWant((H * dk, E)), "v": TensorWant((H * dv, E)),
                "g": TensorWant((H * dv, E)), "a1": TensorWant((self.ra, E)), "a2": TensorWant((H * dk, self.ra)),
                "a2_bias": TensorWant((H * dk,), **keep), "norm": TensorWant((dv,), init="ones_normal", **keep),
                "o": TensorWant((E, H * dv))}

    def state_spec(self):
        return {"S": StateSpec((self.H, self.dk, self.dv), torch.float32)}

    def load(self, tensors) -> None:
        take = lambda n: self._take(tensors, n)
        H, dk, dv = self.H, self.dk, self.dv
        # one product for everything that reads h: [q | k | v | g | a1]
        self.w_in = ops.decode_weight(_fuse([take(n) for n in ("q", "k", "v", "g", "a1")]), "plain",
                                      self.decode_copies)
        self.g_off = 2 * H * dk + H * dv
        self.a_off = self.g_off + H * dv
        self.w_a2 = ops.decode_weight(take("a2").contiguous(), "plain", self.decode_copies)
        self.a2_bias = take("a2_bias").to(torch.float32).contiguous()
        self.norm_w = take("norm").contiguous()
        self.w_o = ops.decode_weight(take("o").contiguous(), "plain", self.decode_copies)

    def tunables(self):
        return (("plain", self.w_o, {}),)

    def forward(self, h, ctx: StepContext, line, writes_cache, position):
        H, dk, dv = self.H, self.dk, self.dv
        U = ops.linear(h, self.w_in)
        Z = ops.linear(U[:, self.a_off:].contiguous(), self.w_a2)
        qn, kn, vv, weight, dec = ops.gla_prepare(U, 0, H * dk, 2 * H * dk, Z, self.a2_bias, self.tau, H, dk, dv)
        S = ctx.cache.state_line(line)["S"]
        o = ops.delta_scan(qn, kn, vv, weight, dec, S, ctx.cu_seqlens, ctx.seq_slot, ctx.n_seqs,
                           ctx.max_rows if ctx.prefill else 1, correct=False)
        y = ops.delta_finish(o, self.norm_w, U, self.g_off, "silu", self.eps, ctx.act_dtype)
        return ops.linear(y, self.w_o)


@register_part("mixer", "lightning_attention")
class LightningAttention(Mixer):
    """Per head a matrix of state S [key_dim, value_dim] with one fixed decay:

        q = silu(W_q h),  k = silu(W_k h),  v = silu(W_v h)
        S <- decay_h S + k v^T;   o = S^T q
        out = W_o (o / rms(o) * norm * sigmoid(W_g h))

    rms over all heads' outputs side by side (`eps`), `norm` of that width.  Kept per sequence: S
    (float32).  A step goes on from whatever the slot holds: single tokens in one launch, many rows
    a sequence in chunks.  The recurrence is float32; the projections take the engine's dtype.
    """

    graph_safe_prompts = True
    takes_continuations = True

    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, value_dim: int, decay: Sequence[float],
                 eps: float, tensors=None):
        super().__init__(tensors)
        if key_dim > 256:
            raise ValueError(f"lightning attention: a key size of {key_dim} is beyond the kernels' limit of 256")
        if len(decay) != int(num_heads) or any(not 0.0 <= float(g) <= 1.0 for g in decay):
            raise ValueError(f"lightning attention: one decay in [0, 1] for each of {num_heads} heads, got {decay!r}")
        self.E, self.H, self.dk, self.dv = int(hidden_size), int(num_heads), int(key_dim), int(value_dim)
        self.eps, self.decay_values, self.decay = float(eps), [float(g) for g in decay], None

    def shapes(self) -> Dict[str, TensorWant]:
        E, H, dk, dv = self.E, self.H, self.dk, self.dv
        return {"q": TensorWant((H * dk, E)), "k": TensorWant((H * dk, E)), "v": TensorWant((H * dv, E)),
                "g": TensorWant((H * dv, E)), "o": TensorWant((E, H * dv)),
                "norm": TensorWant((H * dv,), init="ones_normal", keep_stored=True)}

    def state_spec(self):
        return {"S": StateSpec((self.H, self.dk, self.dv), torch.float32)}

    def load(self, tensors) -> None:
        take = lambda n: self._take(tensors, n)
        H, dk, dv = self.H, self.dk, self.dv
        # one product for everything that reads h: [q | k | v | g]
        self.w_in = ops.decode_weight(_fuse([take(n) for n in ("q", "k", "v", "g")]), "plain", self.decode_copies)
        self.k_off, self.v_off = H * dk, 2 * H * dk
        self.g_off = self.v_off + H * dv
        self.norm_w = take("norm").contiguous()
        self.decay = torch.tensor(self.decay_values, dtype=torch.float32, device=self.norm_w.device)
        self.w_o = ops.decode_weight(take("o").contiguous(), "plain", self.decode_copies)

    def tunables(self):
        return (("plain", self.w_o, {}),)

    def forward(self, h, ctx: StepContext, line, writes_cache, position):
        H, dk, dv = self.H, self.dk, self.dv
        U = ops.linear(h, self.w_in)
        S = ctx.cache.state_line(line)["S"]
        cols = (0, self.k_off, self.v_off)
        if not ctx.prefill:
            o = ops.lightning_step(U, *cols, self.decay, S, ctx.row_slot, H, dk, dv)
        elif ctx.max_rows >= ops.LIGHTNING_CHUNKS_FROM and ops.lightning_chunks_fits(U, *cols, dk, dv):
            o = ops.lightning_chunks(U, *cols, self.decay, S, ctx.cu_seqlens, ctx.seq_slot, ctx.n_seqs,
                                     ctx.max_rows, H, dk, dv)
        else:
            qn, kn, vv, weight, dec = ops.lightning_prepare(U, *cols, self.decay, H, dk, dv)
            o = ops.delta_scan(qn, kn, vv, weight, dec, S, ctx.cu_seqlens, ctx.seq_slot, ctx.n_seqs,
                               ctx.max_rows, correct=False)
        y = ops.group_norm_gate(o, 1, self.norm_w, U, self.g_off, "sigmoid", self.eps, ctx.act_dtype)
        return ops.linear(y, self.w_o)


@register_part("mixer", "retention")
class Retention(Mixer):
    """Per head a matrix of state S [key_dim, value_dim] with one fixed decay:

        q = rot(W_q h),  k = rot(W_k h) key_dim^-1/2,  v = W_v h       rot: the layer's rotary encoding, if any
        S <- decay_h S + k v^T;   o = S^T q
        out = W_o (o / rms(o) * silu(W_g h))

    rms over each head's outputs (`eps`), without a weight.  Kept per sequence: S (float32).  A step
    goes on from whatever the slot holds: single tokens in one launch, many rows a sequence in chunks.
    Rotation and recurrence are float32; the projections take the engine's dtype.
    """

    graph_safe_prompts = True
    takes_continuations = True
    takes_projected = True

    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, value_dim: int, decay: Sequence[float],
                 eps: float, tensors=None):
        super().__init__(tensors)
        if key_dim > 256:
            raise ValueError(f"retention: a key size of {key_dim} is beyond the kernels' limit of 256")
        if len(decay) != int(num_heads) or any(not 0.0 <= float(g) <= 1.0 for g in decay):
            raise ValueError(f"retention: one decay in [0, 1] for each of {num_heads} heads, got {decay!r}")
        self.E, self.H, self.dk, self.dv = int(hidden_size), int(num_heads), int(key_dim), int(value_dim)
        self.eps, self.decay_values, self.decay = float(eps), [float(g) for g in decay], None
        self.k_scale = 1.0 / math.sqrt(self.dk)

    def shapes(self) -> Dict[str, TensorWant]:
        E, H, dk, dv = self.E, self.H, self.dk, self.dv
        return {"q": TensorWant((H * dk, E)), "k": TensorWant((H * dk, E)), "v": TensorWant((H * dv, E)),
                "g": TensorWant((H * dv, E)), "o": TensorWant((E, H * dv))}

    def state_spec(self):
        return {"S": StateSpec((self.H, self.dk, self.dv), torch.float32)}

    def load(self, tensors) -> None:
        take = lambda n: self._take(tensors, n)
        H, dk, dv = self.H, self.dk, self.dv
        # one product for everything that reads h: [q | k | v | g]
        self.w_in = ops.decode_weight(_fuse([take(n) for n in ("q", "k", "v", "g")]), "plain", self.decode_copies)
        self.k_off, self.v_off = H * dk, 2 * H * dk
        self.g_off = self.v_off + H * dv
        self.decay = torch.tensor(self.decay_values, dtype=torch.float32, device=take("q").device)
        self.w_o = ops.decode_weight(take("o").contiguous(), "plain", self.decode_copies)

    def tunables(self):
        return (("plain", self.w_o, {}),)

    def forward(self, h, ctx: StepContext, line, writes_cache, position, projected=None):
        H, dk, dv = self.H, self.dk, self.dv
        table, rot = (None, 0)
        if position is not None:
            if position.pairing != "half":
                raise ValueError("retention: the rotation pairs i with i + rotary_dim / 2")
            table, rot = position.table(ctx.device), position.rotary_dim
        U, at = projected if projected is not None else (ops.linear(h, self.w_in), 0)
        S = ctx.cache.state_line(line)["S"]
        cols = (at, at + self.k_off, at + self.v_off)
        if not ctx.prefill:
            o = ops.retention_step(U, *cols, self.decay, table, rot, self.k_scale, ctx.row_pos, S, ctx.row_slot, H, dk, dv)
        elif ctx.max_rows >= ops.LIGHTNING_CHUNKS_FROM and ops.retention_chunks_fits(U, cols[2], dk, dv):
            qn, kn = ops.retention_prepare(U, *cols, self.decay, table, rot, self.k_scale, ctx.row_pos, H, dk, dv, scan=False)
            o = ops.retention_chunks(qn, kn, U, cols[2], self.decay, S, ctx.cu_seqlens, ctx.seq_slot, ctx.n_seqs,
                                     ctx.max_rows, H, dk, dv)
        else:
            qn, kn, vv, weight, dec = ops.retention_prepare(U, *cols, self.decay, table, rot, self.k_scale, ctx.row_pos,
                                                            H, dk, dv)
            o = ops.delta_scan(qn, kn, vv, weight, dec, S, ctx.cu_seqlens, ctx.seq_slot, ctx.n_seqs, ctx.max_rows,
                               correct=False)
        y = ops.group_norm_gate(o, H, None, U, at + self.g_off, "silu", self.eps, ctx.act_dtype)
        return ops.linear(y, self.w_o)


@register_part("mixer", "time_mix")
class TimeMix(Mixer):
    """Recurrent time mixing with a token shift (an RWKV-style layer).  Each of five projections reads a mix of
    its own of the token's row and the one before it (zeros before the sequence):

        in_s = h + (h_before - h) mu_s                       s of r, k, v, g, w
        r = W_r in_r,  k = W_k in_k,  v = W_v in_v,  w = exp(-exp(W_w2 tanh(W_w1 in_w) + w0))   one a head and channel
        o = (S + diag(u) k v^T)^T r;   S <- diag(w) S + k v^T           the bonus u counts for the current token alone
        out = W_o (o / rms(o) * norm * silu(W_g in_g))

    rms over each head's outputs (`eps`), `norm` of all heads' width.  Kept per sequence: S [dim, dim] a head
    (float32) and the last row h.  A step goes on from whatever the slot holds: single tokens in one launch, many
    rows a sequence in chunks.  Decays, bonus and the state are float32; the mixes and projections take the
    engine's dtype.  A block that mixes single tokens in its own pass (`takes_token_mixes`, `shift`) hands
    `forward` the mixes as `ops.TokenMixes`.
    """

    graph_safe_prompts = True
    takes_continuations = True
    takes_token_mixes = True
    MIXES = ("r", "k", "v", "g", "w")

    def __init__(self, hidden_size: int, num_heads: int, dim: int, decay_rank: int, eps: float, tensors=None):
        super().__init__(tensors)
        if dim > 256:
            raise ValueError(f"time mixing: a head size of {dim} is beyond the kernels' limit of 256")
        if int(decay_rank) <= 0:
            raise ValueError("time mixing: the decays' rank must be positive")
        self.E, self.H, self.d, self.rank, self.eps = int(hidden_size), int(num_heads), int(dim), int(decay_rank), float(eps)

    def shapes(self) -> Dict[str, TensorWant]:
        E, n, R = self.E, self.H * self.d, self.rank
        keep = dict(keep_stored=True)
        return {**{f"mu_{s}": TensorWant((E,), **keep) for s in self.MIXES},
                "r": TensorWant((n, E)), "k": TensorWant((n, E)), "v": TensorWant((n, E)), "g": TensorWant((n, E)),
                "w1": TensorWant((R, E)), "w2": TensorWant((n, R)), "w0": TensorWant((n,), **keep),
                "u": TensorWant((self.H, self.d), **keep), "norm": TensorWant((n,), init="ones_normal", **keep),
                "o": TensorWant((E, n))}

    def state_spec(self):
        return {"S": StateSpec((self.H, self.d, self.d), torch.float32), "tail": StateSpec((1, self.E), None)}

    def load(self, tensors) -> None:
        take = lambda n: self._take(tensors, n)
        f32 = lambda n: take(n).to(torch.float32).contiguous()
        n = self.H * self.d
        self.mu = torch.stack([f32(f"mu_{s}") for s in self.MIXES]).contiguous()
        # one stacked matrix; each part reads rows of its own: [r | k | v | g | w1]
        self.w_in = ops.decode_weight(_fuse([take(t) for t in ("r", "k", "v", "g", "w1")]), "plain", self.decode_copies)
        self.ends = (n, 2 * n, 3 * n, 4 * n, 4 * n + self.rank)
        # (from the tanh on the decays' map is float32 arithmetic: single tokens read the stored rows, steps of
        # several tokens a float32 copy)
        self.w2_rows = take("w2").to(ops.plain_weight(self.w_in).dtype).contiguous()
        self.w_w2 = self.w2_rows.to(torch.float32).contiguous()
        self.w0, self.u, self.norm_w = f32("w0"), f32("u").reshape(-1).contiguous(), take("norm").contiguous()
        self.w_o = ops.decode_weight(take("o").contiguous(), "plain", self.decode_copies)

    def tunables(self):
        return (("plain", self.w_o, {}),)

    def shift(self, ctx: StepContext, line):
        """(mu, tail, row_slot): what a pass that mixes single tokens needs (`ops.post_add_rmsnorm`)."""
        return self.mu, ctx.cache.state_line(line)["tail"], ctx.row_slot

    def forward(self, h, ctx: StepContext, line, writes_cache, position):
        H, d = self.H, self.d
        state = ctx.cache.state_line(line)
        S = state["S"]
        if isinstance(h, ops.TokenMixes):
            planes = h.planes
        else:
            planes = ops.token_mix(h, self.mu, state["tail"], ctx.row_slot, update_tail=not ctx.prefill)
            if ctx.prefill:
                ops.short_conv_tail(h, 0, state["tail"], ctx.cu_seqlens, ctx.seq_slot, ctx.n_seqs, 2)
        r, k, v, g, low = ops.linear_parts(planes, self.w_in, self.ends)
        if not ctx.prefill and self.rank <= ops.TIME_MIX_STEP_MAX_RANK and self.w2_rows.dtype == r.dtype:
            o = ops.time_mix_step(r, k, v, low, self.w2_rows, self.w0, self.u, S, ctx.row_slot, H, d)
        else:
            Z = ops.linear(ops.tanh_rows(low), self.w_w2)
            if ctx.prefill and ctx.max_rows >= ops.TIME_MIX_CHUNKS_FROM and ops.time_mix_chunks_fits(r, k, v, d):
                o = ops.time_mix_chunks(r, k, v, Z, self.w0, self.u, S, ctx.cu_seqlens, ctx.seq_slot, ctx.n_seqs,
                                        ctx.max_rows, H, d)
            else:
                rn, kn, vv, beta, dec = ops.time_mix_prepare(r, k, v, Z, self.w0, self.u, H, d)
                o = ops.delta_scan(rn, kn, vv, beta, dec, S, ctx.cu_seqlens, ctx.seq_slot, ctx.n_seqs,
                                   ctx.max_rows if ctx.prefill else 1, correct="bonus")
        y = ops.group_norm_gate(o, H, self.norm_w, g, 0, "silu", self.eps, ctx.act_dtype)
        return ops.linear(y, self.w_o)


# decay = exp(-rate sigmoid(z)): the rule fixes the rate, so a channel keeps at least exp(-rate) a token
REMOVAL_DECAY_RATE = math.exp(-0.5)


@register_part("mixer", "removal_delta_rule")
class RemovalDeltaRule(Mixer):
    """A generalized delta rule: per head a matrix of state S [dim, dim] whose decay, removal and
    writing each have a vector of their own:

        r = W_r h,  k = W_k h,  v = W_v h,   u = k / sqrt(sum k^2 + 1e-6) a head
        w = exp(-exp(-1/2) sigmoid(W_w2 tanh(W_w1 h) + w0)),   a = sigmoid(W_a h + b_a)     a head and channel
        S_new = diag(w) S - (a u) (u^T S) + k v^T;   o = S_new^T r
        out = W_o (o / rms(o) * norm * sigmoid(W_g h))

    rms over each head's outputs (`eps`), `norm` of all heads' width.  Kept per sequence: S (float32).
    A step goes on from whatever the slot holds: single tokens in one launch, many rows a sequence in
    chunks.  Decays, rates, unit
    keys and the state are float32; the projections take the engine's dtype.
    """

    graph_safe_prompts = True
    takes_continuations = True

    def __init__(self, hidden_size: int, num_heads: int, dim: int, decay_rank: int, eps: float, tensors=None):
        super().__init__(tensors)
        if dim > 256:
            raise ValueError(f"removal delta rule: a head size of {dim} is beyond the kernels' limit of 256")
        if int(decay_rank) <= 0:
            raise ValueError("removal delta rule: the decays' rank must be positive")
        self.E, self.H, self.d, self.rank, self.eps = int(hidden_size), int(num_heads), int(dim), int(decay_rank), float(eps)

    def shapes(self) -> Dict[str, TensorWant]:
        E, n, R = self.E, self.H * self.d, self.rank
        keep = dict(keep_stored=True)
        return {"r": TensorWant((n, E)), "k": TensorWant((n, E)), "v": TensorWant((n, E)), "g": TensorWant((n, E)),
                "a": TensorWant((n, E)), "a_bias": TensorWant((n,), **keep), "w1": TensorWant((R, E)),
                "w2": TensorWant((n, R)), "w0": TensorWant((n,), **keep),
                "norm": TensorWant((n,), init="ones_normal", **keep), "o": TensorWant((E, n))}

    def state_spec(self):
        return {"S": StateSpec((self.H, self.d, self.d), torch.float32)}

    def load(self, tensors) -> None:
        take = lambda n: self._take(tensors, n)
        f32 = lambda n: take(n).to(torch.float32).contiguous()
        n = self.H * self.d
        # one product for everything that reads h: [r | k | v | a | g | w1]
        self.w_in = ops.decode_weight(_fuse([take(t) for t in ("r", "k", "v", "a", "g", "w1")]), "plain",
                                      self.decode_copies)
        self.k_off, self.v_off, self.a_off, self.g_off, self.w1_off = n, 2 * n, 3 * n, 4 * n, 5 * n
        # (the decays' map from the tanh on is float32 arithmetic: single tokens read the stored rows,
        # steps of several tokens a float32 copy)
        self.w2_rows = take("w2").to(ops.plain_weight(self.w_in).dtype).contiguous()
        self.w_w2 = self.w2_rows.to(torch.float32).contiguous()
        self.a_bias, self.w0, self.norm_w = f32("a_bias"), f32("w0"), take("norm").contiguous()
        self.w_o = ops.decode_weight(take("o").contiguous(), "plain", self.decode_copies)

    def tunables(self):
        return (("plain", self.w_o, {}),)

    def forward(self, h, ctx: StepContext, line, writes_cache, position):
        H, d = self.H, self.d
        U = ops.linear(h, self.w_in)
        S = ctx.cache.state_line(line)["S"]
        cols = (0, self.k_off, self.v_off, self.a_off)
        if not ctx.prefill and self.rank <= ops.REMOVAL_STEP_MAX_RANK and self.w2_rows.dtype == U.dtype:
            o = ops.removal_step(U, *cols, self.a_bias, self.w1_off, self.w2_rows, self.w0, REMOVAL_DECAY_RATE, S,
                                 ctx.row_slot, H, d)
        else:
            Z = ops.linear(ops.tanh_columns(U, self.w1_off, self.rank), self.w_w2)
            if ctx.prefill and ctx.max_rows >= ops.REMOVAL_CHUNKS_FROM and d <= ops.REMOVAL_CHUNKS_MAX_DIM:
                o = ops.removal_chunks(U, *cols, self.a_bias, Z, self.w0, REMOVAL_DECAY_RATE, S, ctx.cu_seqlens,
                                       ctx.seq_slot, ctx.n_seqs, ctx.max_rows, H, d)
                return self._finish(o, U, ctx)
            rn, kn, vv, beta, dec, removal = ops.removal_prepare(U, *cols, self.a_bias, Z, self.w0, REMOVAL_DECAY_RATE,
                                                                 H, d)
            o = ops.delta_scan(rn, kn, vv, beta, dec, S, ctx.cu_seqlens, ctx.seq_slot, ctx.n_seqs,
                               ctx.max_rows if ctx.prefill else 1, correct=False, removal=removal)
        return self._finish(o, U, ctx)

    def _finish(self, o, U, ctx: StepContext):
        y = ops.group_norm_gate(o, self.H, self.norm_w, U, self.g_off, "sigmoid", self.eps, ctx.act_dtype)
        return ops.linear(y, self.w_o)


# a = exp(-rate r softplus(lam)): the unit fixes the rate
LRU_RATE = 8.0


@register_part("mixer", "gated_linear_recurrence")
class GatedLinearRecurrence(Mixer):
    """A recurrent block with a real-gated linear recurrent unit.  Two branches `channels` wide:

        y = gelu_tanh(W_y h + b_y)
        u = conv(W_x h + b_x)           a short causal convolution per channel, `conv` taps with a bias,
                                        the last tap on the token itself, zeros ahead of the sequence
        r = sigmoid(R_b u_b + b_r),  i = sigmoid(I_b u_b + b_i)      in `blocks` equal parts b of the
                                        channels, R_b and I_b square [out, in]
        a = exp(-8 r softplus(lam)),   S <- a S + sqrt(1 - a^2) (i u)      from S = 0, one number a channel
        out = W_o (S y)

    Kept per sequence: S (float32) and the convolution's last conv - 1 inputs.  A step goes on from
    whatever the slot holds.  Gates, decays and the state are float32; the projections take the
    engine's dtype.
    """

    graph_safe_prompts = True
    takes_continuations = True

    def __init__(self, hidden_size: int, channels: int, blocks: int, conv: int, tensors=None):
        super().__init__(tensors)
        if int(channels) % int(blocks):
            raise ValueError(f"gated linear recurrence: {channels} channels do not split into {blocks} equal blocks")
        if not 1 <= int(conv) <= 8:
            raise ValueError(f"gated linear recurrence: {conv} taps; the kernels take 1 to 8")
        if int(channels) // int(blocks) > 4096:
            raise ValueError("gated linear recurrence: blocks of more than 4096 channels are beyond the gates' kernel")
        self.E, self.C, self.nb, self.taps = int(hidden_size), int(channels), int(blocks), int(conv)

    def shapes(self) -> Dict[str, TensorWant]:
        E, C, nb = self.E, self.C, self.nb
        cb = C // nb
        keep = dict(keep_stored=True)
        return {"y": TensorWant((C, E)), "y_bias": TensorWant((C,), **keep), "x": TensorWant((C, E)),
                "x_bias": TensorWant((C,), **keep), "conv": TensorWant((C, self.taps), **keep),
                "conv_bias": TensorWant((C,), **keep), "ra": TensorWant((nb, cb, cb), **keep),
                "ra_bias": TensorWant((nb, cb), **keep), "ri": TensorWant((nb, cb, cb), **keep),
                "ri_bias": TensorWant((nb, cb), **keep), "lam": TensorWant((C,), **keep),
                "o": TensorWant((E, C))}

    def state_spec(self):
        return {"S": StateSpec((self.C,), torch.float32),
                "tail": StateSpec((max(self.taps - 1, 1), self.C), None)}

    def load(self, tensors) -> None:
        take = lambda n: self._take(tensors, n)
        f32 = lambda n: take(n).to(torch.float32).contiguous()
        self.w_in = ops.decode_weight(_fuse([take("y"), take("x")]), "plain", self.decode_copies)   # [y | x]
        self.y_bias, self.x_bias = f32("y_bias"), f32("x_bias")
        self.conv_w, self.conv_b = f32("conv"), f32("conv_bias")
        # the gates' maps transposed ([in, out] per block), so that neighbouring threads read
        # neighbouring outputs
        self.w_gates = torch.stack([f32("ra").transpose(1, 2), f32("ri").transpose(1, 2)]).contiguous()
        self.r_bias, self.i_bias = f32("ra_bias").reshape(-1), f32("ri_bias").reshape(-1)
        self.lam = f32("lam")
        self.w_o = ops.decode_weight(take("o").contiguous(), "plain", self.decode_copies)

    def tunables(self):
        return (("plain", self.w_o, {}),)

    def forward(self, h, ctx: StepContext, line, writes_cache, position):
        C = self.C
        U = ops.linear(h, self.w_in)
        state = ctx.cache.state_line(line)
        S, tail = state["S"], state["tail"]
        u = ops.short_conv(U, C, C, self.conv_w, tail, ctx.row_slot, torch.float32, bias=self.conv_b,
                           in_bias=self.x_bias, update_tail=not ctx.prefill)
        if ctx.prefill:
            ops.short_conv_tail(U, C, tail, ctx.cu_seqlens, ctx.seq_slot, ctx.n_seqs, self.taps,
                                in_bias=self.x_bias)
        a, x = ops.lru_gates(u, self.w_gates, self.r_bias, self.i_bias, self.lam, LRU_RATE)
        y = ops.lru_scan(a, x, S, U, 0, self.y_bias, ctx.cu_seqlens, ctx.seq_slot, ctx.n_seqs,
                         ctx.max_rows if ctx.prefill else 1, ctx.act_dtype)
        return ops.linear(y, self.w_o)
