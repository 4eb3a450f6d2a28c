"""A per-layer token input: beside its embedding every token has a short row for every layer,
which a layer mixes into the stream x behind its feed-forward:

    g = gelu(W_gate x) * e,   x <- x + rms(W_proj g) w        e: the layer's piece of table[token]

(gelu in its tanh form; the norm has a plain weight). One table [vocab, layers x dim] serves all
layers. The sum of the stream and what is still to be added to it is formed by the kernel that
hands the stream on in the activation dtype; the norm and its sum are left to the next norm.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..registry import register_part
from ..weights.source import TensorSpec
from .base import NormedRows, NormedSum, Part, PendingRows, StepContext, WeightBinder, plain_rows


class TokenSideTable(Part):
    """The table of all layers' rows, held once for the model."""

    def __init__(self, tensor: str, vocab: int, layers: int, dim: int):
        self.tensor, self.vocab, self.layers, self.dim = tensor, vocab, layers, dim
        self.table: Optional[torch.Tensor] = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        return {self.tensor: TensorSpec((self.vocab, self.layers * self.dim))}

    def bind(self, w: WeightBinder) -> None:
        self.table = w.matrix(self.tensor)


class TokenSide(Part):
    def __init__(self, prefix: str, hidden: int, table: TokenSideTable, layer: int, eps: float,
                 names=("gate", "proj", "norm")):
        """`layer`: which piece of the table's rows this layer reads."""
        if not 0 <= layer < table.layers:
            raise ValueError(f"layer {layer} has no piece of a table for {table.layers} layers")
        self.prefix, self.hidden, self.source, self.layer = prefix, hidden, table, layer
        self.eps, self.names = float(eps), tuple(names)
        self.w_gate: Optional[torch.Tensor] = None
        self.w_proj: Optional[torch.Tensor] = None
        self.gain: Optional[torch.Tensor] = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        p, n, d = self.prefix, self.names, self.source.dim
        return {p + n[0]: TensorSpec((d, self.hidden)), p + n[1]: TensorSpec((self.hidden, d)),
                p + n[2]: TensorSpec((self.hidden,), "gain")}

    def bind(self, w: WeightBinder) -> None:
        self.w_gate, self.w_proj, self.gain = (w.matrix(self.prefix + self.names[0]),
                                               w.matrix(self.prefix + self.names[1]),
                                               w.float32(self.prefix + self.names[2]))

    def forward(self, ctx: StepContext, residual: torch.Tensor, pending) -> NormedRows:
        ops, d = ctx.ops, self.source.dim
        if isinstance(pending, PendingRows):
            pending.add_to(ctx, residual)
            pending = None
        elif isinstance(pending, NormedSum):
            pending = plain_rows(ctx, pending)
        x = ctx.empty((ctx.T, self.hidden))
        ops.stream_norm(residual, pending, out=x)
        z, g = ctx.empty((ctx.T, d)), ctx.empty((ctx.T, d))
        ops.linear(x, self.w_gate, z)
        ops.token_gate(z, self.source.table, ctx.tokens, self.layer * d, g)
        y = ctx.empty((ctx.T, self.hidden))
        ops.linear(g, self.w_proj, y)
        return NormedRows(y, self.gain, self.eps)


register_part("input", "token_side", TokenSide)
