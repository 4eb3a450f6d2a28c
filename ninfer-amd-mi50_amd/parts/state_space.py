"""A state-space layer with a decay per head and token (the mixer of Mamba-2):

    [z | x | B | C | dt] = W_in h       z, x: heads x vdim;  B, C: groups x state;  dt: heads
    [x | B | C] <- silu(conv([x | B | C]) + b)       a causal convolution over time per channel
    dt <- softplus(dt + b_dt)
    S_t = e^(-e^(A) dt) S_(t-1) + dt B_t x_t^T,   y_t = S_t^T C_t + D x_t
          (per head; head h reads B and C of group h // (heads / groups); A, D: a number per head)
    out = W_o ( rms(y silu(z)) * weight )       normed in `norm_groups` equal parts of a row

z, x, B and C are one product; dt is a product of its own with a 32-bit result. dt, the decays, the
recurrence, its state and the norm are 32-bit. The state (S [heads, state, vdim], then the
convolution's last taps - 1 inputs) lives in the request's state slot, starts at zero, and is carried
from step to step; nothing is kept per token.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..registry import register_part
from ..weights.source import TensorSpec
from .base import CallInfo, Mixer, StepContext, WeightBinder


class StateSpace(Mixer):
    def __init__(self, prefix: str, hidden: int, heads: int, vdim: int, state: int, groups: int, taps: int,
                 norm_groups: int, eps: float,
                 names=("in", "conv", "conv.b", "dt_bias", "A_log", "D", "norm", "o")):
        """`names`: what follows the prefix in the tensors' names: the input product [2 heads vdim +
        2 groups state + heads, hidden], the convolution's taps [channels, taps] (the last one the
        row's own) and bias, dt's bias, A, D [heads], the norm's weight [heads * vdim], the output
        product."""
        if heads % groups or (heads * vdim) % norm_groups:
            raise ValueError(f"{heads} heads of {vdim} do not split into {groups} groups or {norm_groups} norm groups")
        if taps < 1:
            raise ValueError(f"a convolution has at least one tap, got {taps}")
        self.prefix, self.names = prefix, tuple(names)
        self.hidden, self.heads, self.vdim, self.state, self.groups = hidden, heads, vdim, state, groups
        self.taps, self.norm_groups, self.eps = taps, norm_groups, float(eps)
        self.inner, self.channels = heads * vdim, heads * vdim + 2 * groups * state
        self.w_in: Optional[torch.Tensor] = None
        self.w_dt: Optional[torch.Tensor] = None
        self.w_o: Optional[torch.Tensor] = None
        self.conv_w: Optional[torch.Tensor] = None     # [taps, channels]: a tap's weights side by side
        self.conv_b: Optional[torch.Tensor] = None
        self.dt_bias: Optional[torch.Tensor] = None
        self.rate: Optional[torch.Tensor] = None       # e^A
        self.skip: Optional[torch.Tensor] = None       # D
        self.norm_w: Optional[torch.Tensor] = None

    def _memory_floats(self) -> int:
        # (whole pieces of 16 bytes)
        return -(-self.heads * self.state * self.vdim // 4) * 4

    def state_floats(self) -> int:
        return self._memory_floats() + -(-(self.taps - 1) * self.channels // 4) * 4

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        p, n, H = self.prefix, self.names, self.heads
        return {p + n[0]: TensorSpec((self.inner + self.channels + H, self.hidden)),
                p + n[1]: TensorSpec((self.channels, self.taps), "gain"),
                p + n[2]: TensorSpec((self.channels,), "bias"), p + n[3]: TensorSpec((H,), "bias"),
                p + n[4]: TensorSpec((H,), "bias"), p + n[5]: TensorSpec((H,), "gain"),
                p + n[6]: TensorSpec((self.inner,), "gain"), p + n[7]: TensorSpec((self.hidden, self.inner))}

    def bind(self, w: WeightBinder) -> None:
        p, n = self.prefix, self.names
        whole = w.matrix(p + n[0])
        self.w_in, self.w_dt = whole[:self.inner + self.channels], whole[self.inner + self.channels:]
        taps = w.float32(p + n[1])
        self.conv_w = taps.t().contiguous()
        w.hold(p + n[1], self.conv_w.t())
        self.conv_b = w.float32(p + n[2])
        self.dt_bias = w.float32(p + n[3])
        self.rate = torch.exp(w.float32(p + n[4]))     # (read-back by name hands out A itself)
        self.skip = w.float32(p + n[5])
        self.norm_w = w.float32(p + n[6])
        self.w_o = w.matrix(p + n[7])

    def forward(self, ctx: StepContext, x, residual, call: CallInfo):
        ops, inner, n = ctx.ops, self.inner, self._memory_floats()
        u = ctx.empty((ctx.T, inner + self.channels))
        dt = ctx.empty((ctx.T, self.heads), torch.float32)
        with ops.together():
            ops.linear(x, self.w_in, u)
            ops.linear(x, self.w_dt, dt)
        xbc = ctx.empty((ctx.T, self.channels))
        ops.conv_silu(u[:, inner:], self.conv_w, self.conv_b, call.state[:, n:], ctx, xbc)
        y = ctx.empty((ctx.T, inner), torch.float32)
        ops.state_space(xbc, self.heads, self.vdim, self.state, self.groups, dt, self.dt_bias, self.rate, self.skip,
                        call.state[:, :n], ctx, y)
        normed = ctx.empty((ctx.T, inner))
        ops.gated_rmsnorm(y, u[:, :inner], self.norm_w, self.eps, normed, group=inner // self.norm_groups,
                          gate_act="silu", gate_first=True)
        out = ctx.empty((ctx.T, self.hidden))
        ops.linear(normed, self.w_o, out)
        return out


register_part("mixer", "state_space", StateSpace)
