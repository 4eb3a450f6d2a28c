"""A matrix memory with exponential gates (the mLSTM of xLSTM), one per head:

    q = W_q h dim^(-1/2), k = W_k h   (heads x dim),   v = W_v h   (heads x vdim)
    i = c(W_i h + b_i),  f = log_sigmoid(c(W_f h + b_f)),  c(z) = cap tanh(z / cap)     (per head)
    m_t = max(f_t + m_(t-1), i_t)                                  (a running maximum, from 0)
    S_t = e^(f_t + m_(t-1) - m_t) S_(t-1) + e^(i_t - m_t) k_t v_t^T,   z_t alike with k_t alone
    o_t = S_t^T q_t / (max(|z_t . q_t|, e^(-m_t)) + 1e-6)
    y = W_o ( concat_heads(rms_vdim(o_t)) * weight * sigmoid(W_g h) )

The wide input products are one product over the stacked weight [2 H dim + 2 H vdim, hidden]
(q, k, v, gate), which mixers side by side may share; the gates' logits are a product of their own
with a 32-bit result. The gates, the recurrence, its state and the norm are 32-bit. The state (S
[heads, dim, vdim], then z [heads, dim], then m [heads]) lives in the request's state slot, starts at
zero, and is carried from step to step; nothing is kept per token.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..registry import register_part
from ..weights.source import TensorSpec
from .base import CallInfo, Mixer, StepContext, WeightBinder


class MatrixMemory(Mixer):
    def __init__(self, prefix: str, hidden: int, heads: int, dim: int, vdim: int, cap: float, eps: float,
                 q_scale: Optional[float] = None,
                 names=("q", "k", "v", "g", "o", "i", "f", "i.b", "f.b", "norm")):
        """`cap`: the bound on both gates' logits. `q_scale`: the factor on q (None:
        dim^(-1/2)). `names`: what follows the prefix in the names of W_q, W_k, W_v, W_g, W_o, W_i,
        W_f, the gates' biases [heads] and the norm's weight [heads * vdim]."""
        if not cap > 0:
            raise ValueError(f"cap ({cap}) must be positive")
        self.prefix, self.names = prefix, tuple(names)
        self.hidden, self.heads, self.dim, self.vdim = hidden, heads, dim, vdim
        self.cap, self.eps = float(cap), float(eps)
        self.q_scale = float(q_scale) if q_scale is not None else dim ** -0.5
        self.shares_input = False
        self.w_in: Optional[torch.Tensor] = None
        self.w_o: Optional[torch.Tensor] = None
        self.w_gates: Optional[torch.Tensor] = None
        self.b_gates: Optional[torch.Tensor] = None
        self.norm_w: Optional[torch.Tensor] = None

    def state_floats(self) -> int:
        # (whole pieces of 16 bytes, so that every request's state starts at one)
        return -(-self.heads * (self.dim * self.vdim + self.dim + 1) // 4) * 4

    def _widths(self):
        qk, v = self.heads * self.dim, self.heads * self.vdim
        return qk, qk, v, v

    def input_width(self) -> int:
        return sum(self._widths())

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        p, n, H = self.prefix, self.names, self.heads
        specs = {p + name: TensorSpec((width, self.hidden)) for name, width in zip(n[:4], self._widths())}
        specs.update({p + n[4]: TensorSpec((self.hidden, H * self.vdim)), p + n[5]: TensorSpec((H, self.hidden)),
                      p + n[6]: TensorSpec((H, self.hidden)), p + n[7]: TensorSpec((H,), "bias"),
                      p + n[8]: TensorSpec((H,), "bias"), p + n[9]: TensorSpec((H * self.vdim,), "gain")})
        return specs

    def bind_input(self, w: WeightBinder, rows: torch.Tensor) -> None:
        at = 0
        for name, width in zip(self.names[:4], self._widths()):
            w.matrix_into(self.prefix + name, rows[at:at + width])
            at += width

    def bind(self, w: WeightBinder) -> None:
        p, n, H = self.prefix, self.names, self.heads
        if not self.shares_input:
            self.w_in = torch.empty((self.input_width(), self.hidden), dtype=w.act_dtype, device=w.device)
            self.bind_input(w, self.w_in)
        self.w_o = w.matrix(p + n[4])
        self.w_gates = torch.empty((2 * H, self.hidden), dtype=w.act_dtype, device=w.device)
        w.matrix_into(p + n[5], self.w_gates[:H])
        w.matrix_into(p + n[6], self.w_gates[H:])
        self.b_gates = torch.cat([w.float32(p + n[7]), w.float32(p + n[8])])
        w.hold(p + n[7], self.b_gates[:H])
        w.hold(p + n[8], self.b_gates[H:])
        self.norm_w = w.float32(p + n[9])

    def input_extra(self, ctx: StepContext, x):
        gates = ctx.empty((ctx.T, 2 * self.heads), torch.float32)
        ctx.ops.linear(x, self.w_gates, gates)
        return gates

    def mix_projected(self, ctx: StepContext, u, call: CallInfo, extra=None):
        qk, v = self.heads * self.dim, self.heads * self.vdim
        out = ctx.empty((ctx.T, v))
        ctx.ops.matrix_memory(u, 0, qk, 2 * qk, extra, self.b_gates, self.heads, self.dim, self.vdim, self.cap,
                              self.q_scale, call.state, ctx, u[:, 2 * qk + v:], self.norm_w, self.eps, out)
        return out

    def output(self, ctx: StepContext, rows):
        out = ctx.empty((ctx.T, self.hidden))
        ctx.ops.linear(rows, self.w_o, out)
        return out

    def forward(self, ctx: StepContext, x, residual, call: CallInfo):
        u = ctx.empty((ctx.T, self.input_width()))
        with ctx.ops.together():
            ctx.ops.linear(x, self.w_in, u)
            extra = self.input_extra(ctx, x)
        return self.forward_projected(ctx, u, call, extra)


register_part("mixer", "matrix_memory", MatrixMemory)
