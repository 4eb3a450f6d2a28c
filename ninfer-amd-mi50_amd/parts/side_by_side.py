"""Two mixers side by side on the same input, in one of two forms:

    y = factor (rms(left(h)) g_l + rms(right(h)) g_r)      (each output normed over the model
                                                            width with a gain per column of its own)
    y = left_factor left(h) + right_factor right(h)         (no norms)

Both read h through one shared product (their `input_width`s side by side), and the norms and
the sum are left to whoever takes the result (`NormedSum`, `SumRows`): a block's norm kernel forms
them on the fly. In steps of many rows the right mixer runs on the second stream beside the left
one. The cache is the one mixer's that asks for pages; the state holds the left one's, then the
right one's.
"""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..registry import register_part
from ..weights.source import TensorSpec
from .base import (CacheNeed, CallInfo, Mixer, NormedSum, Part, StepContext, SumRows,
                   WeightBinder)


class SideBySide(Mixer):
    def __init__(self, left: Mixer, right: Mixer, left_norm: Optional[str] = None,
                 right_norm: Optional[str] = None, hidden: int = 0, eps: float = 0.0,
                 factor: float = 0.5, left_factor: float = 1.0, right_factor: float = 1.0):
        """`left_norm`, `right_norm`: the names of the outputs' gains [hidden] (both or neither;
        the first form with, the second without them)."""
        if left.input_width() is None or right.input_width() is None:
            raise ValueError("mixers side by side read their input through one product each")
        if left.cache_need() is not None and right.cache_need() is not None:
            raise ValueError("two mixers side by side that both keep pages are not built")
        if (left_norm is None) != (right_norm is None):
            raise ValueError("both outputs are normed or neither")
        if left_norm is not None and (left_factor != 1.0 or right_factor != 1.0):
            raise ValueError("a factor on each of two normed outputs is not built")
        self.left, self.right = left, right
        self.left_norm, self.right_norm = left_norm, right_norm
        self.hidden, self.eps, self.factor = hidden, float(eps), float(factor)
        self.left_factor, self.right_factor = float(left_factor), float(right_factor)
        left.shares_input = right.shares_input = True
        self.w_in: Optional[torch.Tensor] = None
        self.gain_l: Optional[torch.Tensor] = None
        self.gain_r: Optional[torch.Tensor] = None

    def children(self) -> List[Part]:
        return [self.left, self.right]

    def cache_need(self) -> Optional[CacheNeed]:
        need = self.left.cache_need()
        return need if need is not None else self.right.cache_need()

    def state_floats(self) -> int:
        return self.left.state_floats() + self.right.state_floats()

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        return {n: TensorSpec((self.hidden,), "gain") for n in (self.left_norm, self.right_norm) if n}

    def bind(self, w: WeightBinder) -> None:
        a, b = self.left.input_width(), self.right.input_width()
        self.w_in = torch.empty((a + b, self.hidden), dtype=w.act_dtype, device=w.device)
        self.left.bind_input(w, self.w_in[:a])
        self.right.bind_input(w, self.w_in[a:])
        if self.left_norm:
            self.gain_l, self.gain_r = w.float32(self.left_norm), w.float32(self.right_norm)

    def _call(self, call: CallInfo, mixer: Mixer, at: int) -> CallInfo:
        n = mixer.state_floats()
        return CallInfo(cache=call.cache if mixer.cache_need() is not None else None,
                        writes_cache=call.writes_cache, state=call.state[:, at:at + n] if n else None)

    def forward(self, ctx: StepContext, x, residual, call: CallInfo):
        ops, a = ctx.ops, self.left.input_width()
        u = ctx.empty((ctx.T, self.w_in.shape[0]))
        with ops.together():
            ops.linear(x, self.w_in, u)
            extra_l, extra_r = self.left.input_extra(ctx, x), self.right.input_extra(ctx, x)
        to_left = self._call(call, self.left, 0)
        to_right = self._call(call, self.right, self.left.state_floats())
        if ops.wants_beside(ctx.T):
            with ops.beside():
                y_r = self.right.forward_projected(ctx, u[:, a:], to_right, extra_r)
            y_l = self.left.forward_projected(ctx, u[:, :a], to_left, extra_l)
            ops.join()
        else:
            l = self.left.mix_projected(ctx, u[:, :a], to_left, extra_l)
            r = self.right.mix_projected(ctx, u[:, a:], to_right, extra_r)
            with ops.together():
                y_l, y_r = self.left.output(ctx, l), self.right.output(ctx, r)
        if self.left_norm is None:
            return SumRows(y_l, self.left_factor, y_r, self.right_factor)
        return NormedSum(y_l, self.gain_l, y_r, self.gain_r, self.eps, self.factor)


register_part("mixer", "side_by_side", SideBySide)
