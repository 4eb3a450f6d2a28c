"""Typed configuration of Nosedra, a decoder-only model whose layers are listed one by one.

config.json keys: `architecture` ("Nosedra"), `vocab`, `width`, `norm.eps`, `logit_softcap`
(absent or 0: logits are not capped), `token_side.dim` (numbers per layer of the table of
per-layer token inputs), and `layers`: a list of objects with `type` ('parallel' or 'mamba2'),
`mixer` (sizes and constants) and `mlp` (null, or {'kind': 'dense', 'ff'}).
A parallel mixer has `left` {`heads`, `kv_heads`, `dim`, `vdim`, `scale`, `rot` {`base`, `dims`,
`scaling` {`factor`}}} (`kv_heads` absent: as many as heads; `vdim` absent: dim; `rot` absent: no
rotation; `scaling` absent: plain frequencies), `right` {`heads`, `dim`, `vdim`, `gate_cap`},
`left_scale` and `right_scale`. A mamba2 mixer has `heads`, `vdim`, `state`, `groups`, `conv` (taps)
and `norm_groups`.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from .base import ConfigError, KeyReader


@dataclass(frozen=True)
class RotaryConfig:
    dims: int                 # how many numbers of a head turn (0: none)
    base: float
    factor: float             # every frequency is divided by it


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: RotaryConfig


@dataclass(frozen=True)
class MatrixMemoryConfig:
    heads: int
    dim: int
    vdim: int
    gate_cap: float


@dataclass(frozen=True)
class ParallelConfig:
    left: AttentionConfig
    right: MatrixMemoryConfig
    left_scale: float
    right_scale: float


@dataclass(frozen=True)
class Mamba2Config:
    heads: int
    vdim: int
    state: int
    groups: int
    taps: int
    norm_groups: int


@dataclass(frozen=True)
class NosedraLayer:
    type: str                 # 'parallel' | 'mamba2'
    mixer: Any
    ff: Optional[int]         # inner size of the feed-forward (None: the layer has none)


@dataclass(frozen=True)
class NosedraConfig:
    vocab: int
    width: int
    eps: float
    softcap: float
    side_dim: int
    layers: Tuple[NosedraLayer, ...]
    architecture: str = "Nosedra"

    @staticmethod
    def from_dict(raw: Dict[str, Any]) -> "NosedraConfig":
        r = KeyReader(raw)
        vocab = r.need_int("vocab", 1)
        width = r.need_int("width", 1)
        eps = _positive(_sub(r, "norm"), "eps")
        softcap = r.opt_float("logit_softcap", 0.0)
        if softcap < 0:
            raise ConfigError(f"config.json: key 'logit_softcap' must be >= 0, got {softcap}")
        side = _sub(r, "token_side").need_int("dim", 1)
        entries = r.opt_raw("layers")
        if not isinstance(entries, list) or not entries:
            raise ConfigError("config.json: key 'layers' must be a non-empty list")
        return NosedraConfig(vocab, width, eps, softcap, side,
                             tuple(_layer(x, i) for i, x in enumerate(entries)))


def _sub(r: KeyReader, key: str) -> KeyReader:
    v = r.opt_raw(key)
    if not isinstance(v, dict):
        raise ConfigError(f"{r.where}: key '{key}' must be an object")
    return KeyReader(v, f"{r.where}: {key}")


def _positive(r: KeyReader, key: str) -> float:
    v = r.need_float(key)
    if not v > 0:
        raise ConfigError(f"{r.where}: key '{key}' must be > 0, got {v}")
    return v


def _rot(m: KeyReader, most: int) -> RotaryConfig:
    if m.opt_raw("rot") is None:
        return RotaryConfig(0, 10000.0, 1.0)
    rot = _sub(m, "rot")
    dims = rot.opt_int("dims", most, 0)
    if dims % 2 or dims > most:
        raise ConfigError(f"{rot.where}: 'rot.dims' must be even and at most {most}, got {dims}")
    base = _positive(rot, "base")
    factor = 1.0
    if rot.opt_raw("scaling") is not None:
        factor = _positive(_sub(rot, "scaling"), "factor")
    return RotaryConfig(dims, base, factor)


def _attention(m: KeyReader) -> AttentionConfig:
    heads = m.need_int("heads", 1)
    kv_heads = m.opt_int("kv_heads", heads, 1)
    if heads % kv_heads:
        raise ConfigError(f"{m.where}: 'heads' must be a multiple of 'kv_heads'")
    dim = m.need_int("dim", 1)
    return AttentionConfig(heads, kv_heads, dim, m.opt_int("vdim", dim, 1), _positive(m, "scale"), _rot(m, dim))


def _memory(m: KeyReader) -> MatrixMemoryConfig:
    dim = m.need_int("dim", 1)
    return MatrixMemoryConfig(m.need_int("heads", 1), dim, m.opt_int("vdim", dim, 1), _positive(m, "gate_cap"))


def _mamba2(m: KeyReader) -> Mamba2Config:
    c = Mamba2Config(m.need_int("heads", 1), m.need_int("vdim", 1), m.need_int("state", 1),
                     m.opt_int("groups", 1, 1), m.need_int("conv", 1), m.opt_int("norm_groups", 1, 1))
    if c.heads % c.groups:
        raise ConfigError(f"{m.where}: 'heads' must be a multiple of 'groups'")
    if c.heads * c.vdim % c.norm_groups:
        raise ConfigError(f"{m.where}: 'norm_groups' must divide heads x vdim")
    return c


def _layer(entry: Any, i: int) -> NosedraLayer:
    where = f"config.json: layers[{i}]"
    if not isinstance(entry, dict):
        raise ConfigError(f"{where} must be an object")
    r = KeyReader(entry, where)
    kind = r.opt_str("type", None)
    m = _sub(r, "mixer")
    if kind == "parallel":
        mixer = ParallelConfig(_attention(_sub(m, "left")), _memory(_sub(m, "right")),
                               m.need_float("left_scale"), m.need_float("right_scale"))
    elif kind == "mamba2":
        mixer = _mamba2(m)
    else:
        raise ConfigError(f"{where}: 'type' must be 'parallel' or 'mamba2', got {kind!r}")
    ff = None
    if r.opt_raw("mlp") is not None:
        f = _sub(r, "mlp")
        fk = f.opt_str("kind", "dense")
        if fk != "dense":
            raise ConfigError(f"{where}: 'mlp.kind' must be 'dense', got {fk!r}")
        ff = f.need_int("ff", 1)
    return NosedraLayer(kind, mixer, ff)
