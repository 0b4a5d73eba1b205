"""Two mixers that read the same rows; their outputs are added with a scale each."""
from __future__ import annotations

from typing import Dict

import torch

from ..kernels import ops
from ..weights.loader import TensorWant
from .base import Mixer, StepContext, build_part, register_part


@register_part("mixer", "side_by_side")
class SideBySide(Mixer):
    """out = left_scale * left(h) + right_scale * right(h).

    `left` and `right` are `PartSpec`s of mixers.  The pair keeps on its cache line what its
    mixers keep: at most one of them keys and values, at most one fixed-size state.  A block that
    adds scaled sums in a kernel of its own sets `takes_scaled_sums` and gets the two outputs as
    `ops.ScaledSum`; any other gets their float32 sum.

    With `norm_size` each output first passes an RMS norm of its own over that width (`norm_eps`; tensors
    `left_norm`, `right_norm`), and the two scales are one and the same.  A block that forms that in a kernel
    of its own sets `takes_normed_pairs` and gets the pieces as `ops.NormedPair`.

    Mixers that both read their input through one stacked matrix (`Mixer.takes_projected`) get theirs stacked
    into one: a single product makes the columns of both.

    `left_position`, `right_position`: `PartSpec`s of position encodings of the mixers' own, in place of the
    block's.
    """

    takes_scaled_sums = False
    takes_normed_pairs = False

    def __init__(self, left, right, left_scale: float = 1.0, right_scale: float = 1.0, norm_size: int = 0,
                 norm_eps: float = 1e-6, left_position=None, right_position=None, tensors=None):
        super().__init__(tensors)
        self.left, self.right = build_part("mixer", left), build_part("mixer", right)
        self.left_scale, self.right_scale = float(left_scale), float(right_scale)
        both = (self.left, self.right)
        self.norm_size, self.norm_eps = int(norm_size), float(norm_eps)
        if self.norm_size and self.left_scale != self.right_scale:
            raise ValueError("side_by_side: outputs with norms of their own have one scale")
        self.own_positions = [build_part("position", p) if p is not None else None for p in (left_position, right_position)]
        self.norms = self.w_in = None
        self.right_column = 0
        if sum(m.kv_spec() is not None for m in both) > 1 or sum(m.state_spec() is not None for m in both) > 1:
            raise ValueError("side_by_side: a cache line holds one mixer's keys and values and one "
                             "mixer's state; these two both keep the same kind")
        self.graph_safe = all(m.graph_safe for m in both)
        self.graph_safe_prompts = all(m.graph_safe_prompts for m in both)
        self.takes_continuations = all(m.takes_continuations for m in both)

    def wants(self) -> Dict[str, TensorWant]:
        return {**super().wants(), **self.left.wants(), **self.right.wants()}

    def shapes(self) -> Dict[str, TensorWant]:
        norm = lambda: TensorWant((self.norm_size,), init="ones_normal", keep_stored=True)
        return {"left_norm": norm(), "right_norm": norm()} if self.norm_size else {}

    def kv_spec(self):
        return self.left.kv_spec() or self.right.kv_spec()

    def state_spec(self):
        return self.left.state_spec() or self.right.state_spec()

    def load(self, tensors) -> None:
        for m, own in zip((self.left, self.right), self.own_positions):
            m.decode_copies, m.position = self.decode_copies, own if own is not None else self.position
            m.load(tensors)
        if self.left.takes_projected and self.right.takes_projected:
            a, b = ops.plain_weight(self.left.w_in), ops.plain_weight(self.right.w_in)
            if a.dtype == b.dtype:
                # (rows of zeros up to a multiple of 8, so that the right mixer's columns are as aligned as alone)
                pad = a.new_zeros((-a.shape[0] % 8, a.shape[1]))
                self.right_column = a.shape[0] + pad.shape[0]
                self.w_in = ops.decode_weight(torch.cat([a, pad, b], dim=0).contiguous(), "plain", self.decode_copies)
                self.left.w_in = self.right.w_in = None
        if self.norm_size:
            self.norms = [self._take(tensors, n).contiguous() for n in ("left_norm", "right_norm")]

    def tunables(self):
        return tuple(self.left.tunables()) + tuple(self.right.tunables())

    def forward(self, h, ctx: StepContext, line, writes_cache, position):
        of_left, of_right = (own if own is not None else position for own in self.own_positions)
        of_both = ({}, {})
        if self.w_in is not None:
            U = ops.linear(h, self.w_in)
            of_both = ({"projected": (U, 0)}, {"projected": (U, self.right_column)})
        a = self.left.forward(h, ctx, line, writes_cache, of_left, **of_both[0])
        b = self.right.forward(h, ctx, line, writes_cache, of_right, **of_both[1])
        if self.norm_size:
            pair = ops.NormedPair(a, self.norms[0], b, self.norms[1], self.norm_eps, self.left_scale)
            return pair if self.takes_normed_pairs else pair.tensor()
        both = ops.ScaledSum(a, self.left_scale, b, self.right_scale)
        return both if self.takes_scaled_sums else both.tensor()
