"""What every part of a model is: its interface and the data a step hands it.

A model is put together from parts: a mixer (attention here), a feed-forward
(dense or experts), norms, a position encoding, and a block that arranges
them. A part has its sizes and constants as constructor parameters, names the
checkpoint tensors it needs, and runs on the rows of one step. No part knows
which model it is in: it sees its own parameters, a name prefix, and a
`StepContext`.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional, Tuple

import torch

from ..weights.source import TensorSpec


@dataclass(frozen=True)
class PoolSpec:
    """One paged pool of a mixer: what it keeps per token under `name`.

    The pool's tensor is [pages, *outer, page_size, *inner]: `outer` are the
    dimensions a page is split by before its token slots (heads, for keys and
    values), `inner` what one token holds in one of them (a head's numbers).
    `dtype` None means the engine's activation dtype; 'float32' or 'bfloat16'
    fix it."""
    name: str
    outer: Tuple[int, ...]
    inner: Tuple[int, ...]
    dtype: Optional[str] = None

    def elements_per_token(self) -> int:
        n = 1
        for d in self.outer + self.inner:
            n *= d
        return n


@dataclass(frozen=True)
class CacheNeed:
    """What a mixer needs of the paged cache for each token it has seen: any
    number of named pools, each with a per-token shape and dtype of its own,
    for all positions (window None) or only the last `window` of them, in pages
    of `page_size` tokens (None: the engine's). Mixers with the same window and
    page size share page numbers and block tables; each has pools of its own.

    `stride` > 1: an entry of the pools belongs to a whole block of `stride` tokens (block b to
    positions b stride .. (b + 1) stride - 1; it exists once all of them are cached), and a page
    holds `page_size` such entries. `blocks`: a second need of the same mixer, with names of
    its own, kept in a group (page numbers, block tables) of its own: what it keeps per block of
    tokens beside what it keeps per token."""
    pools: Tuple[PoolSpec, ...]
    window: Optional[int] = None
    page_size: Optional[int] = None
    stride: int = 1
    blocks: Optional["CacheNeed"] = None

    def all_needs(self) -> Tuple["CacheNeed", ...]:
        return (self,) if self.blocks is None else (self, self.blocks)

    def bytes_per_token(self, bytes_per_element: int) -> int:
        """Bytes of the pools per token (those of blocks: their share of one token, rounded
        up); pools without a dtype of their own count `bytes_per_element` per number."""
        own = {"float32": 4, "bfloat16": 2}
        return sum(-(-sum(p.elements_per_token() * (own[p.dtype] if p.dtype else bytes_per_element)
                          for p in n.pools) // n.stride) for n in self.all_needs())

    @staticmethod
    def keys_values(kv_heads: int, head_dim: int, window: Optional[int] = None,
                    page_size: Optional[int] = None, vdim: Optional[int] = None,
                    block: Optional[int] = None) -> "CacheNeed":
        """Keys and values of `kv_heads` heads of `head_dim` (values: `vdim`, when given):
        pools 'k' [pages, kv_heads, page_size, head_dim] and 'v' [.., vdim]; with `block` also
        one key and value for every whole block of so many tokens, of all positions: pools
        'k_block' and 'v_block' of the same shapes."""
        def pair(suffix):
            return (PoolSpec("k" + suffix, (kv_heads,), (head_dim,)),
                    PoolSpec("v" + suffix, (kv_heads,), (head_dim if vdim is None else vdim,)))
        blocks = CacheNeed(pair("_block"), None, page_size, stride=block) if block else None
        return CacheNeed(pair(""), window, page_size, blocks=blocks)


@dataclass
class CacheView:
    """One cache instance as a step sees it: the mixer's pools by name (each
    [pages, *outer, page_size, *inner]) and the block table of the step's
    requests [S, max_pages] (int32, -1 where a page was given back). `blocks`: the same for
    what the mixer keeps per block of `stride` tokens, when it keeps any."""
    pools: Dict[str, torch.Tensor]
    block_table: torch.Tensor
    page_size: int
    window: Optional[int]
    stride: int = 1
    blocks: Optional["CacheView"] = None

    def __getitem__(self, name: str) -> torch.Tensor:
        return self.pools[name]


@dataclass
class CallInfo:
    """How one entry of the layer plan runs: which cache it uses, whether it
    writes it (false when it reads another call's cache), and the slice of the
    per-request state that belongs to it ([slots, floats], or None): a block's for the block,
    the mixer's for the mixer."""
    cache: Optional[CacheView] = None
    writes_cache: bool = True
    state: Optional[torch.Tensor] = None


@dataclass
class StepContext:
    """The rows of one step and what parts need to run them.

    T rows of S requests; rows of one request are contiguous and in order.
    All index tensors are int32 on the device. `host` holds the same numbers as
    Python lists for sizing launches without a device round trip.
    """
    ops: Any
    act_dtype: torch.dtype
    device: torch.device
    T: int
    S: int
    tokens: torch.Tensor          # [T]
    positions: torch.Tensor       # [T] absolute position of each row in its request
    row_seq: torch.Tensor         # [T] index (within this step) of the row's request
    seq_slots: torch.Tensor       # [S] slot of each request (index into state)
    seq_row_start: torch.Tensor   # [S + 1] first row of each request, then T
    seq_qlen: torch.Tensor        # [S]
    seq_pos0: torch.Tensor        # [S] position of the request's first row
    max_qlen: int = 1
    max_kv_len: int = 1
    all_decode: bool = False
    single_rows: int = 0          # the first single_rows requests bring one row each (rows 0 ..)
    scratch: Dict[str, Any] = field(default_factory=dict)

    def empty(self, shape, dtype=None) -> torch.Tensor:
        return torch.empty(shape, dtype=dtype or self.act_dtype, device=self.device)


@dataclass
class PendingRows:
    """A weighted sum of rows that a part leaves to be added to the residual by
    whoever comes next (a norm's kernel adds it on the fly):
    sum_j weights[t, j] * y[t * k + j, :] + sigmoid(gate[t]) * shared[t, :].
    `shared` and `gate` may be None (no such term / factor 1). `gate` is a
    32-bit view [T] that may be strided. With `ids` ([T, k], the chosen experts), a choice j
    with ids[t, j] >= `real` stands for an expert without weights that hands its input back:
    its term is weights[t, j] * rows[t, :] (`rows`: what the experts read), and row t * k + j
    of y holds nothing."""
    y: torch.Tensor
    weights: torch.Tensor
    shared: Optional[torch.Tensor] = None
    gate: Optional[torch.Tensor] = None
    ids: Optional[torch.Tensor] = None
    real: int = 0
    rows: Optional[torch.Tensor] = None

    def add_to(self, ctx: "StepContext", residual: torch.Tensor) -> None:
        if self.ids is not None:
            ctx.ops.gated_sum_add(residual, None, None, None, self, None, None, 1.0)
        else:
            ctx.ops.moe_combine(residual, self.y, self.weights, self.shared, self.gate)


@dataclass
class NormedSum:
    """Rows that a mixer leaves to be formed by whoever comes next:
    factor * (rms(a) gain_a + rms(b) gain_b) with rms(y) = y rsqrt(mean(y^2) + eps), from rows
    a, b [T, hidden] and gains [hidden] (32-bit)."""
    a: torch.Tensor
    gain_a: torch.Tensor
    b: torch.Tensor
    gain_b: torch.Tensor
    eps: float
    factor: float

    def rows(self, ctx: "StepContext") -> torch.Tensor:
        """The rows themselves, for parts that take only plain ones."""
        total = torch.zeros(self.a.shape, dtype=torch.float32, device=self.a.device)
        ctx.ops.norm_add(total, self.a, self.gain_a * self.factor, self.eps)
        ctx.ops.norm_add(total, self.b, self.gain_b * self.factor, self.eps)
        return total.to(ctx.act_dtype)


@dataclass
class ReadyRows:
    """Nothing is left to be added to the residual; `rows` is the residual in the activation
    dtype, for a block that reads it as it is."""
    rows: torch.Tensor


@dataclass
class SumRows:
    """Rows that a part leaves to be added to the residual by whoever comes next, in 32-bit:
    factor_a a + factor_b b + bias, from rows a and b [T, hidden] (b may be None) and a bias
    [hidden] (32-bit, or None)."""
    a: torch.Tensor
    factor_a: float = 1.0
    b: Optional[torch.Tensor] = None
    factor_b: float = 1.0
    bias: Optional[torch.Tensor] = None

    def rows(self, ctx: "StepContext") -> torch.Tensor:
        """The rows themselves, for parts that take only plain ones."""
        return _formed(ctx, self, self.a)


@dataclass
class NormedRows:
    """The same for rows that are normed first: y rsqrt(mean(y^2) + eps) gain, gain [hidden]
    (32-bit)."""
    y: torch.Tensor
    gain: torch.Tensor
    eps: float

    def rows(self, ctx: "StepContext") -> torch.Tensor:
        return _formed(ctx, self, self.y)


def _formed(ctx: "StepContext", pending, like: torch.Tensor) -> torch.Tensor:
    total = torch.zeros(like.shape, dtype=torch.float32, device=like.device)
    ctx.ops.stream_norm(total, pending)
    return total.to(ctx.act_dtype)


def plain_rows(ctx: "StepContext", y):
    """What a part handed on as something that any part takes: a NormedSum, a SumRows or a
    NormedRows becomes rows, a ReadyRows nothing; everything else is handed back unchanged."""
    if isinstance(y, (NormedSum, SumRows, NormedRows)):
        return y.rows(ctx)
    return None if isinstance(y, ReadyRows) else y


def settle(ctx: "StepContext", residual: torch.Tensor, pending) -> Optional[torch.Tensor]:
    """For parts that take only plain rows: a PendingRows is added into the
    residual now; a tensor (or None) is handed back unchanged."""
    if isinstance(pending, PendingRows):
        pending.add_to(ctx, residual)
        return None
    return plain_rows(ctx, pending)


class WeightBinder:
    """Reads tensors by name from a weight source and places them on the
    device: matrices in the compute dtype, gains and biases in 32-bit. It keeps
    a record name -> the device tensor (or the slice of a fused or stacked one)
    that now holds that checkpoint tensor, so that what the engine holds can be
    read back by checkpoint name."""

    def __init__(self, source: Any, device: torch.device, act_dtype: torch.dtype):
        self.source = source
        self.device = device
        self.act_dtype = act_dtype
        self.held: Dict[str, torch.Tensor] = {}

    def hold(self, name: str, where: torch.Tensor) -> None:
        """Record (or correct, after a part has moved it) where a tensor lives."""
        self.held[name] = where

    def matrix(self, name: str) -> torch.Tensor:
        t = self.source.read(name).to(device=self.device, dtype=self.act_dtype).contiguous()
        self.held[name] = t
        return t

    def float32(self, name: str) -> torch.Tensor:
        t = self.source.read(name).to(device=self.device, dtype=torch.float32).contiguous()
        self.held[name] = t
        return t

    def matrix_into(self, name: str, out: torch.Tensor) -> None:
        """Copy a matrix into a slice of a larger (fused or stacked) tensor."""
        out.copy_(self.source.read(name).to(device=self.device), non_blocking=False)
        self.held[name] = out


class Part:
    """Base of all parts. `prefix` is the part's checkpoint name prefix."""

    prefix: str = ""

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        """Full checkpoint names this part needs -> expected shape and role."""
        return {}

    def unused_tensor_specs(self) -> Dict[str, TensorSpec]:
        """Checkpoint names that may be there and that this part does not read
        (a copy of a tied table, a stored table of constants): present with the
        shape given they are passed over, absent they are not missed."""
        return {}

    def bind(self, w: WeightBinder) -> None:
        """Read this part's tensors (fusing or stacking them as its kernels
        want them)."""

    def children(self) -> List["Part"]:
        return []

    def max_positions(self) -> Optional[int]:
        """The most positions a request may have because of this part (a table of learned
        positions has so many rows), or None: no limit of its own. The engine refuses a
        `max_context` beyond the least of its parts' limits."""
        return None

    def least_max_positions(self) -> Optional[int]:
        limits = [self.max_positions()] + [c.least_max_positions() for c in self.children()]
        limits = [x for x in limits if x is not None]
        return min(limits) if limits else None

    def all_tensor_specs(self) -> Dict[str, TensorSpec]:
        out = dict(self.tensor_specs())
        for c in self.children():
            out.update(c.all_tensor_specs())
        return out

    def all_unused_tensor_specs(self) -> Dict[str, TensorSpec]:
        out = dict(self.unused_tensor_specs())
        for c in self.children():
            out.update(c.all_unused_tensor_specs())
        return out

    def bind_all(self, w: WeightBinder) -> None:
        self.bind(w)
        for c in self.children():
            c.bind_all(w)


class Norm(Part):
    """y = norm(residual [+ pending]); the sum is kept in `residual` (32-bit).
    `pending` is rows [T, hidden], a PendingRows, or None (a norm that cannot
    add a PendingRows on the fly calls `settle` first)."""

    def forward(self, ctx: StepContext, residual: torch.Tensor,
                pending: Optional[torch.Tensor]) -> torch.Tensor:
        raise NotImplementedError

    def forward_rows(self, ctx: StepContext, residual: torch.Tensor, rows: torch.Tensor,
                     pending: Optional[torch.Tensor] = None) -> torch.Tensor:
        """Norm of selected rows of residual [+ pending]; `residual` is left as
        it is."""
        raise NotImplementedError


class PositionEncoding(Part):
    """A position encoding applied to queries and keys inside a mixer: a
    rotation of the first `rot_dim` dims of every head, pair i by the angle
    pos * table()[i]. `pairing` says which dims form pair i: 'half' pairs
    (i, i + rot_dim / 2), 'interleaved' the neighbours (2i, 2i + 1). The table
    holds any frequencies (scaled per dimension or not); rot_dim 0 is no
    rotation."""

    rot_dim: int = 0
    pairing: str = "half"

    def table(self) -> Optional[torch.Tensor]:
        raise NotImplementedError


class Mixer(Part):
    """Mixes information between the positions of a request.

    `cache_need()` says what it keeps per token in pages (None: nothing; else
    named pools, each with its own per-token shape and dtype),
    `state_floats()` how many 32-bit numbers of fixed-size state it keeps per
    request (0: none). `forward` takes the normed rows [T, hidden] and returns
    rows [T, hidden] that the block adds to the residual.
    """

    def cache_need(self) -> Optional[CacheNeed]:
        return None

    def state_floats(self) -> int:
        return 0

    def input_width(self) -> Optional[int]:
        """Columns of the one product through which this mixer reads its input, or None when it
        reads it in another way. A mixer that gives a width also has `bind_input(w, rows)`
        (place the product's weights into `rows` [input_width, hidden]) and
        `mix_projected(ctx, u, call, extra)` (`u`: the product's [T, input_width], columns of a
        wider row-major tensor; returns what `output` takes), so that mixers which read the same
        input share one product; its own `bind` then leaves these weights alone once
        `shares_input` is set."""
        return None

    def input_extra(self, ctx: StepContext, x: torch.Tensor):
        """Small products of the input that stay beside the shared one (numbers wanted in
        32-bit): called inside `together()`, handed to `mix_projected` as `extra`."""
        return None

    def mix_projected(self, ctx: StepContext, u: torch.Tensor, call: CallInfo, extra=None) -> torch.Tensor:
        raise NotImplementedError

    def output(self, ctx: StepContext, rows: torch.Tensor) -> torch.Tensor:
        """The output product of what `mix_projected` returned."""
        raise NotImplementedError

    def forward_projected(self, ctx: StepContext, u: torch.Tensor, call: CallInfo, extra=None) -> torch.Tensor:
        return self.output(ctx, self.mix_projected(ctx, u, call, extra))

    def forward(self, ctx: StepContext, x: torch.Tensor, residual: torch.Tensor,
                call: CallInfo) -> Optional[torch.Tensor]:
        raise NotImplementedError


class FeedForward(Part):
    """Row-wise transform. `forward` returns what is to be added to the
    residual: rows [T, hidden], a PendingRows, or None if it has already added
    its result to `residual` itself."""

    def forward(self, ctx: StepContext, x: torch.Tensor, residual: torch.Tensor
                ) -> Optional[torch.Tensor]:
        raise NotImplementedError


class Block(Part):
    """Arrangement of norms, mixer and feed-forward around the residual."""

    mixer: Mixer

    def state_floats(self) -> int:
        """32-bit numbers of per-request state of one run of this block: the mixer's, and
        whatever the block's other parts keep (a block that has such parts adds them and hands
        each its columns of `CallInfo.state`)."""
        return self.mixer.state_floats()

    def forward(self, ctx: StepContext, residual: torch.Tensor,
                pending: Optional[torch.Tensor], call: CallInfo) -> Optional[torch.Tensor]:
        raise NotImplementedError
