"""Nosedra put together from parts, layer by layer from its configuration.

x = embed[token]; every layer is pre-norm (norm gains stored around zero),
    x <- x + mixer(rms(x) (1 + w1)),   x <- x + ff(rms(x) (1 + w2)),
    x <- x + rms(side.proj (gelu(side.gate x) * e)) w   with e the layer's part of side.embed[token]
where the mixer is two mixers side by side on the same input, their outputs added with a factor
each (causal attention with rotated, then unit-normed queries and keys, a learned sink per head
and an output gate; a matrix memory with exponential gates), or a state-space layer with a decay
per head and token behind a short convolution. The feed-forward, when the layer has one, is gated
by the tanh form of gelu and has biases. logits = cap tanh(head (rms(x) (1 + w)) / cap).
Tensor names: embed, side.embed, head, final.norm, and per layer l<i>.{norm1, norm2, mix.left.{q, k,
v, g, o, sink} and mix.right.{q, k, v, g, o, i, i.b, f, f.b, norm} or mix.{in, conv, conv.b, dt_bias,
A_log, D, norm, o}, mlp.{gate, up, down} and their .b, side.{gate, proj, norm}}.
"""
from __future__ import annotations

from .. import parts  # noqa: F401  (registers the part factories by kind and name)
from ..config.nosedra import AttentionConfig, NosedraConfig
from ..parts.embedding import LMHead, TokenEmbedding
from ..parts.token_side import TokenSideTable
from ..registry import make_part, register_architecture
from .spec import ModelSpec

_NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "g": "g", "sink": "sink"}


def _attention(m: AttentionConfig, prefix: str, cfg: NosedraConfig):
    if m.rot.dims:
        position = make_part("position", "rotary", rot_dim=m.rot.dims, theta=m.rot.base,
                             scaling={"factor": m.rot.factor})
    else:
        position = make_part("position", "none")
    return make_part("mixer", "attention", prefix=prefix, hidden=cfg.width, heads=m.heads,
                     kv_heads=m.kv_heads, head_dim=m.dim, vdim=m.vdim, position=position,
                     qkv_bias=False, scale=m.scale, qk_norm="unit", qk_norm_eps=cfg.eps,
                     sink="learned", output_gate=True, names=_NAMES)


def build_nosedra(cfg: NosedraConfig) -> ModelSpec:
    w = cfg.width
    table = TokenSideTable("side.embed", cfg.vocab, len(cfg.layers), cfg.side_dim)
    blocks = []
    for i, layer in enumerate(cfg.layers):
        p, m = f"l{i}.", layer.mixer
        if layer.type == "parallel":
            right = make_part("mixer", "matrix_memory", prefix=p + "mix.right.", hidden=w, heads=m.right.heads,
                              dim=m.right.dim, vdim=m.right.vdim, cap=m.right.gate_cap, eps=cfg.eps)
            mixer = make_part("mixer", "side_by_side", left=_attention(m.left, p + "mix.left.", cfg), right=right,
                              hidden=w, left_factor=m.left_scale, right_factor=m.right_scale)
        else:
            mixer = make_part("mixer", "state_space", prefix=p + "mix.", hidden=w, heads=m.heads, vdim=m.vdim,
                              state=m.state, groups=m.groups, taps=m.taps, norm_groups=m.norm_groups, eps=cfg.eps)
        ff = None
        if layer.ff is not None:
            ff = make_part("feed_forward", "swiglu", prefix=p + "mlp.", hidden=w, inner=layer.ff,
                           act="gelu_pytorch_tanh", bias=True, names=("gate", "up", "down"),
                           bias_names=("gate.b", "up.b", "down.b"), hand_on_bias=True)
        norms = [make_part("norm", "rmsnorm", prefix=p + n, size=w, eps=cfg.eps, leaf="", around_zero=True)
                 for n in ("norm1", "norm2")]
        side = make_part("input", "token_side", prefix=p + "side.", hidden=w, table=table, layer=i, eps=cfg.eps)
        blocks.append(make_part("block", "pre_norm", mixer_norm=norms[0], mixer=mixer, ff_norm=norms[1],
                                feed_forward=ff, after=side))
    return ModelSpec(TokenEmbedding("embed", cfg.vocab, w, leaf=""), blocks,
                     make_part("norm", "rmsnorm", prefix="final.norm", size=w, eps=cfg.eps, leaf="",
                               around_zero=True),
                     LMHead("head", cfg.vocab, w, leaf="", softcap=cfg.softcap), shared=[table])


register_architecture("Nosedra", NosedraConfig.from_dict, build_nosedra)
