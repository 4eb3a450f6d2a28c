"""Linear attention whose forget gate also decides what is written (no keys of its own).

    q = silu(W_q h)   (heads x dim),   v = W_v h   (heads x vdim)
    f = l + (1 - l) sigmoid(W_f h + b)             (heads x dim; l: a lower bound per channel)
    S_t = diag(f_t) S_(t-1) + (1 - f_t) v_t^T,   o_t = S_t^T q_t          (per head)
    y = W_o concat_heads(rmsnorm_vdim(o_t) * weight)

The recurrence is the second form of the gated linear attention kernels. The three input
products are one product over the stacked weight [2 H dim + H vdim, hidden] (q, f, v), which
mixers side by side may share. The gate, the recurrence, its state and the norm are 32-bit. The
state S ([heads, dim, vdim] per request) lives in the request's state slot, starts at zero, and
is carried from step to step; nothing is kept per token.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..registry import register_part
from ..weights.source import TensorSpec
from .base import CallInfo, Mixer, StepContext, WeightBinder


class ForgetGateAttention(Mixer):
    def __init__(self, prefix: str, hidden: int, heads: int, dim: int, vdim: int, eps: float,
                 q_scale: float = 1.0, names=("q", "f", "v", "o", "f.b", "lower", "norm")):
        """`names`: what follows the prefix in the names of W_q, W_f, W_v, W_o, the gate's bias
        and lower bounds [heads * dim] and the norm's weight [vdim]. `q_scale`: a factor on q."""
        self.prefix, self.names = prefix, tuple(names)
        self.hidden, self.heads, self.dim, self.vdim = hidden, heads, dim, vdim
        self.eps, self.q_scale = float(eps), float(q_scale)
        self.shares_input = False
        self.w_in: Optional[torch.Tensor] = None
        self.w_o: Optional[torch.Tensor] = None
        self.f_bias: Optional[torch.Tensor] = None
        self.lower: Optional[torch.Tensor] = None
        self.norm_w: Optional[torch.Tensor] = None

    def state_floats(self) -> int:
        return self.heads * self.dim * self.vdim

    def input_width(self) -> int:
        return self.heads * (2 * self.dim + self.vdim)

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        p, n = self.prefix, self.names
        qk, v = self.heads * self.dim, self.heads * self.vdim
        return {p + n[0]: TensorSpec((qk, self.hidden)), p + n[1]: TensorSpec((qk, self.hidden)),
                p + n[2]: TensorSpec((v, self.hidden)), p + n[3]: TensorSpec((self.hidden, v)),
                p + n[4]: TensorSpec((qk,), "bias"), p + n[5]: TensorSpec((qk,), "unit"),
                p + n[6]: TensorSpec((self.vdim,), "gain")}

    def bind_input(self, w: WeightBinder, rows: torch.Tensor) -> None:
        qk = self.heads * self.dim
        for i, (a, b) in enumerate(((0, qk), (qk, 2 * qk), (2 * qk, self.input_width()))):
            w.matrix_into(self.prefix + self.names[i], rows[a:b])

    def bind(self, w: WeightBinder) -> None:
        p, n = self.prefix, self.names
        if not self.shares_input:
            self.w_in = torch.empty((self.input_width(), self.hidden), dtype=w.act_dtype, device=w.device)
            self.bind_input(w, self.w_in)
        self.w_o = w.matrix(p + n[3])
        self.f_bias = w.float32(p + n[4])
        self.lower = w.float32(p + n[5])
        self.norm_w = w.float32(p + n[6])
        if not bool(((self.lower >= 0) & (self.lower <= 1)).all()):
            raise ValueError(f"{p + n[5]}: a forget gate's lower bounds lie between 0 and 1")

    def mix_projected(self, ctx: StepContext, u, call: CallInfo, extra=None):
        ops = ctx.ops
        qk, v = self.heads * self.dim, self.heads * self.vdim
        o = ctx.empty((ctx.T, v), torch.float32)
        # (a step with prompt portions runs in chunks, which keep their scaled rows here)
        wf = ops.gla_work_floats(u.dtype, ctx, self.heads, self.dim)
        work = ctx.empty((ctx.T, wf), torch.float32) if wf else None
        ops.gated_linear_attention(u, 0, 0, 2 * qk, None, self.heads, self.dim, self.vdim, 1.0,
                                   self.q_scale, call.state, ctx, o, work=work,
                                   forget=(qk, self.f_bias, self.lower))
        normed = ctx.empty((ctx.T, v))
        ops.gated_rmsnorm(o, None, self.norm_w, self.eps, normed, group=self.vdim)
        return normed

    def output(self, ctx: StepContext, rows):
        out = ctx.empty((ctx.T, self.hidden))
        ctx.ops.linear(rows, self.w_o, out)
        return out

    def forward(self, ctx: StepContext, x, residual, call: CallInfo):
        u = ctx.empty((ctx.T, self.input_width()))
        ctx.ops.linear(x, self.w_in, u)
        return self.forward_projected(ctx, u, call)


register_part("mixer", "forget_gate_attention", ForgetGateAttention)
