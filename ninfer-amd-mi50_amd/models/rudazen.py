"""Rudazen put together from parts, layer by layer from its configuration.

x = embed[token] scale; every layer norms the stream behind its sums,
    x <- rms(alpha x + mixer(x)) w1,   x <- rms(alpha x + ff(x)) w2
where the mixer is attention over a window whose values are the projected keys, with queries
and keys normed over their whole projections before they turn in neighbouring pairs, and with
the mean key and value of every block of tokens before the window in the same softmax; or two
mixers side by side, each output normed, half their sum: windowed attention with grouped
key/value heads (whole-projection norms, half-split pairs at ramped frequencies, a factor per
head on the scores, a gate on the output) and linear attention whose forget gate decides what
is written. The feed-forward, when the layer has one, is a SwiGLU. logits = head rms(x) w.
Tensor names: embed, head, final.norm, and per layer l<i>.{norm1, norm2, mix.{q, k, o, q.norm,
k.norm} or mix.left.{q, k, v, o, g, q.norm, k.norm, temp, out} and mix.right.{q, f, f.b,
lower, v, norm, o, out}, mlp.{gate, up, down}}.
"""
from __future__ import annotations

from .. import parts  # noqa: F401  (registers the part factories by kind and name)
from ..config.rudazen import AttentionConfig, RotaryConfig, RudazenConfig
from ..parts.embedding import LMHead, TokenEmbedding
from ..registry import make_part, register_architecture
from .spec import ModelSpec

# fixed by the design: two mixers side by side count half each
SIDE_FACTOR = 0.5
_NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "g": "g", "temp": "temp", "q_norm": "q.norm",
          "k_norm": "k.norm"}


def _position(rot: RotaryConfig, pairing: str):
    if not rot.dims:
        return make_part("position", "none")
    s = rot.scaling
    return make_part("position", "rotary", rot_dim=rot.dims, theta=rot.base, pairing=pairing,
                     scaling=None if s is None else {"factor": s.factor, "original": s.original,
                                                     "fast": s.fast, "slow": s.slow})


def _attention(m: AttentionConfig, prefix: str, cfg: RudazenConfig, pairing: str, **more):
    return make_part("mixer", "attention", prefix=prefix, hidden=cfg.width, heads=m.heads,
                     kv_heads=m.kv_heads, head_dim=m.dim, vdim=m.vdim,
                     position=_position(m.rot, pairing), qkv_bias=False, window=m.window,
                     scale=m.scale, qk_norm_eps=cfg.eps, qk_norm="projection", names=_NAMES, **more)


def build_rudazen(cfg: RudazenConfig) -> ModelSpec:
    w = cfg.width
    blocks = []
    for i, layer in enumerate(cfg.layers):
        p, m = f"l{i}.", layer.mixer
        if layer.type == "attention":
            mixer = _attention(m, p + "mix.", cfg, "interleaved", values="keys", pool=m.pool)
        else:
            left = _attention(m.left, p + "mix.left.", cfg, "half", head_temp=True, output_gate=True)
            right = make_part("mixer", "forget_gate_attention", prefix=p + "mix.right.", hidden=w,
                              heads=m.right.heads, dim=m.right.dim, vdim=m.right.vdim, eps=cfg.eps)
            mixer = make_part("mixer", "side_by_side", left=left, right=right,
                              left_norm=p + "mix.left.out", right_norm=p + "mix.right.out", hidden=w,
                              eps=cfg.eps, factor=SIDE_FACTOR)
        ff = None
        if layer.ff is not None:
            ff = make_part("feed_forward", "swiglu", prefix=p + "mlp.", hidden=w, inner=layer.ff,
                           names=("gate", "up", "down"))
        norms = [make_part("norm", "residual_rmsnorm", tensor=p + n, size=w, eps=cfg.eps, alpha=cfg.alpha)
                 for n in ("norm1", "norm2")]
        blocks.append(make_part("block", "post_norm", mixer=mixer, mixer_norm=norms[0],
                                feed_forward=ff, ff_norm=norms[1]))
    return ModelSpec(TokenEmbedding("embed", cfg.vocab, w, leaf="", scale=cfg.embedding_scale), blocks,
                     make_part("norm", "rmsnorm", prefix="final.norm", size=w, eps=cfg.eps, leaf=""),
                     LMHead("head", cfg.vocab, w, leaf=""))


register_architecture("Rudazen", RudazenConfig.from_dict, build_rudazen)
