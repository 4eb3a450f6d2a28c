"""Typed configuration of Rudazen, a decoder-only model whose layers are listed one by one.

config.json keys: `architecture` ("Rudazen"), `vocab`, `width`, `norm.eps`, `postln_alpha` (the
residual's factor in front of every norm), `embedding.scale`, and `layers`: a list of objects
with `type` ('attention' or 'parallel'), `mixer` (sizes and constants) and `mlp` (null, or
{'kind': 'dense', 'ff'}).
An attention mixer has `heads`, `kv_heads`, `dim`, `vdim`, `scale`, `rot` {`base`, `dims`,
`scaling` {`factor`, `original`, `fast`, `slow`}} (absent: no rotation; `scaling` absent: plain
frequencies) and `mask` {`size`, `pool`} (`size` absent: every earlier position; `pool`: tokens
of a block whose mean is seen once it lies before the window; absent: none). A parallel mixer
has `left`, such an attention without `pool`, and `right` {`heads`, `dim`, `vdim`}.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from .base import ConfigError, KeyReader


@dataclass(frozen=True)
class RampScaling:
    factor: float
    original: float
    fast: float
    slow: float


@dataclass(frozen=True)
class RotaryConfig:
    dims: int                 # how many numbers of a head turn (0: none)
    base: float
    scaling: Optional[RampScaling]


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: RotaryConfig
    window: Optional[int]
    pool: Optional[int]       # tokens of a block (None: no blocks)


@dataclass(frozen=True)
class ForgetGateConfig:
    heads: int
    dim: int
    vdim: int


@dataclass(frozen=True)
class ParallelConfig:
    left: AttentionConfig
    right: ForgetGateConfig


@dataclass(frozen=True)
class RudazenLayer:
    type: str                 # 'attention' | 'parallel'
    mixer: Any
    ff: Optional[int]         # inner size of the feed-forward (None: the layer has none)


@dataclass(frozen=True)
class RudazenConfig:
    vocab: int
    width: int
    eps: float
    alpha: float
    embedding_scale: float
    layers: Tuple[RudazenLayer, ...]
    architecture: str = "Rudazen"

    @staticmethod
    def from_dict(raw: Dict[str, Any]) -> "RudazenConfig":
        r = KeyReader(raw)
        vocab = r.need_int("vocab", 1)
        width = r.need_int("width", 1)
        eps = _sub(r, "norm").need_float("eps")
        if not eps > 0:
            raise ConfigError(f"config.json: key 'norm.eps' must be > 0, got {eps}")
        alpha = r.need_float("postln_alpha")
        scale = 1.0
        if r.opt_raw("embedding") is not None:
            scale = _sub(r, "embedding").opt_float("scale", 1.0)
        entries = r.opt_raw("layers")
        if not isinstance(entries, list) or not entries:
            raise ConfigError("config.json: key 'layers' must be a non-empty list")
        return RudazenConfig(vocab, width, eps, alpha, scale,
                             tuple(_layer(x, i) for i, x in enumerate(entries)))


def _sub(r: KeyReader, key: str) -> KeyReader:
    v = r.opt_raw(key)
    if not isinstance(v, dict):
        raise ConfigError(f"{r.where}: key '{key}' must be an object")
    return KeyReader(v, f"{r.where}: {key}")


def _rot(m: KeyReader, most: int) -> RotaryConfig:
    if m.opt_raw("rot") is None:
        return RotaryConfig(0, 10000.0, None)
    rot = _sub(m, "rot")
    dims = rot.opt_int("dims", most, 0)
    if dims % 2 or dims > most:
        raise ConfigError(f"{rot.where}: 'rot.dims' must be even and at most {most}, got {dims}")
    base = rot.need_float("base")
    if not base > 0:
        raise ConfigError(f"{rot.where}: 'rot.base' must be > 0, got {base}")
    scaling = None
    if rot.opt_raw("scaling") is not None:
        s = _sub(rot, "scaling")
        scaling = RampScaling(s.need_float("factor"), s.need_float("original"), s.need_float("fast"),
                              s.need_float("slow"))
        if min(scaling.factor, scaling.original, scaling.fast, scaling.slow) <= 0 or not base > 1:
            raise ConfigError(f"{rot.where}: 'rot.scaling' needs positive numbers and a base above 1")
    return RotaryConfig(dims, base, scaling)


def _attention(m: KeyReader, pools: bool) -> AttentionConfig:
    heads = m.need_int("heads", 1)
    kv_heads = m.opt_int("kv_heads", heads, 1)
    if heads % kv_heads:
        raise ConfigError(f"{m.where}: 'heads' must be a multiple of 'kv_heads'")
    dim = m.need_int("dim", 1)
    vdim = m.opt_int("vdim", dim, 1)
    if pools and vdim != dim:
        raise ConfigError(f"{m.where}: values are keys: 'vdim' ({vdim}) must equal 'dim' ({dim})")
    scale = m.need_float("scale")
    if not scale > 0:
        raise ConfigError(f"{m.where}: 'scale' must be > 0, got {scale}")
    window = pool = None
    if m.opt_raw("mask") is not None:
        mask = _sub(m, "mask")
        window = mask.opt_int("size", None, 1)
        pool = mask.opt_int("pool", None, 1)
        if pool is not None and (not pools or window is None):
            raise ConfigError(f"{mask.where}: 'mask.pool' goes with 'mask.size', in layers of type 'attention'")
    return AttentionConfig(heads, kv_heads, dim, vdim, scale, _rot(m, dim), window, pool)


def _layer(entry: Any, i: int) -> RudazenLayer:
    where = f"config.json: layers[{i}]"
    if not isinstance(entry, dict):
        raise ConfigError(f"{where} must be an object")
    r = KeyReader(entry, where)
    kind = r.opt_str("type", None)
    m = _sub(r, "mixer")
    if kind == "attention":
        mixer = _attention(m, True)
    elif kind == "parallel":
        right = _sub(m, "right")
        mixer = ParallelConfig(_attention(_sub(m, "left"), False), ForgetGateConfig(
            right.need_int("heads", 1), right.need_int("dim", 1), right.need_int("vdim", 1)))
    else:
        raise ConfigError(f"{where}: 'type' must be 'attention' or 'parallel', got {kind!r}")
    ff = None
    if r.opt_raw("mlp") is not None:
        f = _sub(r, "mlp")
        fk = f.opt_str("kind", "dense")
        if fk != "dense":
            raise ConfigError(f"{where}: 'mlp.kind' must be 'dense', got {fk!r}")
        ff = f.need_int("ff", 1)
    return RudazenLayer(kind, mixer, ff)
