"""Rudazen in plain 64-bit arithmetic: one function per mechanism, whole sequences, no cache.

The oracle of the Rudazen tests. It shares no code with the engine: weights come as a dict
name -> tensor, the configuration as the dict that config.json holds. Notation: h is what a
sublayer reads; rms(x) = x / sqrt(mean(x^2) + eps) * w.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

D = torch.float64


def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w.to(D)


def lin(w: Dict[str, torch.Tensor], name: str, x: torch.Tensor) -> torch.Tensor:
    return x @ w[name].to(D).T


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def frequencies(rot: dict) -> Tuple[torch.Tensor, float]:
    """(f_i = base^(-2i / dims) for i < dims / 2, factor on cosine and sine). With `scaling`,
    the pairs that turn least over the original context are slowed down by `factor`, those
    that turn most are kept, and a ramp over the pair's index lies between."""
    dims = rot["dims"]
    f = [rot["base"] ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return torch.tensor(f, dtype=D), 1.0

    def index_of(turns):
        return dims * math.log(sc["original"] / (turns * 2 * math.pi)) / (2 * math.log(rot["base"]))

    lo = max(math.floor(index_of(sc["fast"])), 0)
    hi = min(math.ceil(index_of(sc["slow"])), dims - 1)
    width = max(hi - lo, 0.001)
    out = []
    for i, x in enumerate(f):
        r = min(max((i - lo) / width, 0.0), 1.0)
        out.append(x / sc["factor"] * r + x * (1 - r))
    return torch.tensor(out, dtype=D), 1.0 + 0.1 * math.log(sc["factor"])


def rotate(x: torch.Tensor, pos: torch.Tensor, rot: Optional[dict], pairing: str) -> torch.Tensor:
    """x [n, heads, d]: the first rot.dims numbers of every head turn by pos * f_i; pair i is
    (2i, 2i + 1) when `pairing` is 'interleaved', (i, i + dims / 2) when 'half'."""
    dims = (rot or {}).get("dims", 0)
    if not dims:
        return x
    f, mag = frequencies(rot)
    ang = pos.to(D)[:, None] * f[None, :]
    c, s = mag * torch.cos(ang)[:, None, :], mag * torch.sin(ang)[:, None, :]
    out = x.clone()
    if pairing == "interleaved":
        a, b = slice(0, dims, 2), slice(1, dims, 2)
    else:
        a, b = slice(0, dims // 2), slice(dims // 2, dims)
    u, v = x[..., a], x[..., b]
    out[..., a] = u * c - v * s
    out[..., b] = v * c + u * s
    return out


def visible(n: int, window: Optional[int]) -> torch.Tensor:
    """[n, n] bool: row i sees column j when 0 <= i - j (< window, when there is one)."""
    i = torch.arange(n)[:, None]
    j = torch.arange(n)[None, :]
    m = j <= i
    return m if window is None else m & (i - j < window)


def visible_blocks(n: int, window: int, pool: int) -> torch.Tensor:
    """[n, n // pool] bool: row i sees block b when the block's last token, b pool + pool - 1,
    is at most i - window."""
    i = torch.arange(n)[:, None]
    last = torch.arange(n // pool)[None, :] * pool + pool - 1
    return last <= i - window


def block_means(x: torch.Tensor, pool: int) -> torch.Tensor:
    """x [n, heads, d] -> the means of its whole blocks of `pool` rows [n // pool, heads, d]."""
    nb = x.shape[0] // pool
    return x[:nb * pool].reshape(nb, pool, *x.shape[1:]).mean(1)


def attend(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, window: Optional[int],
           pool: Optional[int] = None, temp: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Softmax attention of q [n, H, d] over k [n, G, d], v [n, G, dv] within the window, and
    with `pool` over the means of the blocks that lie before it, in one softmax. `temp` [H]:
    a factor on each head's scores. Returns [n, H, dv]."""
    n, H = q.shape[:2]
    per = H // k.shape[1]
    vis = visible(n, window)
    if pool:
        vis = torch.cat([visible_blocks(n, window, pool), vis], 1)
        k, v = torch.cat([block_means(k, pool), k]), torch.cat([block_means(v, pool), v])
    out = torch.zeros(n, H, v.shape[-1], dtype=D)
    for a in range(H):
        s = q[:, a] @ k[:, a // per].T * scale
        if temp is not None:
            s = s * temp[a].to(D)
        s = torch.where(vis, s, torch.full((), -math.inf, dtype=D))
        out[:, a] = torch.softmax(s, -1) @ v[:, a // per]
    return out


def pooled_attention(w, p: str, m: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    """The mixer 'attention': values are the projected keys, before norm and rotation."""
    n, H, d = h.shape[0], m["heads"], m["dim"]
    G = m.get("kv_heads", H)
    pos = torch.arange(n)
    q, k = lin(w, p + "q", h), lin(w, p + "k", h)
    v = k.reshape(n, G, d)
    q = rotate(rms_norm(q, w[p + "q.norm"], eps).reshape(n, H, d), pos, m.get("rot"), "interleaved")
    k = rotate(rms_norm(k, w[p + "k.norm"], eps).reshape(n, G, d), pos, m.get("rot"), "interleaved")
    mask = m.get("mask") or {}
    o = attend(q, k, v, m["scale"], mask.get("size"), mask.get("pool"))
    return lin(w, p + "o", o.reshape(n, -1))


def gated_attention(w, p: str, m: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    """The left one of two mixers side by side: window attention with a factor per head on the
    scores and a gate on the output."""
    n, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    G = m.get("kv_heads", H)
    pos = torch.arange(n)
    q = rotate(rms_norm(lin(w, p + "q", h), w[p + "q.norm"], eps).reshape(n, H, d), pos, m.get("rot"), "half")
    k = rotate(rms_norm(lin(w, p + "k", h), w[p + "k.norm"], eps).reshape(n, G, d), pos, m.get("rot"), "half")
    v = lin(w, p + "v", h).reshape(n, G, dv)
    o = attend(q, k, v, m["scale"], (m.get("mask") or {}).get("size"), temp=w[p + "temp"])
    return lin(w, p + "o", o.reshape(n, -1) * torch.sigmoid(lin(w, p + "g", h)))


def forget_gates(z: torch.Tensor, lower: torch.Tensor) -> torch.Tensor:
    lo = lower.to(D)
    return lo + (1 - lo) * torch.sigmoid(z)


def gated_recurrence(q: torch.Tensor, f: torch.Tensor, v: torch.Tensor,
                     state: Optional[torch.Tensor] = None) -> Tuple[torch.Tensor, torch.Tensor]:
    """S_t = diag(f_t) S_(t-1) + (1 - f_t) v_t^T, o_t = S_t^T q_t per head, row by row.
    q, f [n, H, d], v [n, H, dv]; returns (o [n, H, dv], the last state [H, d, dv])."""
    n, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=D) if state is None else state.to(D)
    o = torch.zeros(n, H, v.shape[-1], dtype=D)
    for t in range(n):
        S = f[t][:, :, None] * S + (1 - f[t])[:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    return o, S


def forget_gate_attention(w, p: str, m: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    """The right one of two mixers side by side: linear attention whose forget gate also says
    how much is written."""
    n, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = silu(lin(w, p + "q", h)).reshape(n, H, d)
    f = forget_gates(lin(w, p + "f", h) + w[p + "f.b"].to(D), w[p + "lower"]).reshape(n, H, d)
    v = lin(w, p + "v", h).reshape(n, H, dv)
    o, _ = gated_recurrence(q, f, v)
    return lin(w, p + "o", rms_norm(o, w[p + "norm"], eps).reshape(n, -1))


def side_by_side(w, p: str, m: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    a = gated_attention(w, p + "left.", m["left"], h, eps)
    b = forget_gate_attention(w, p + "right.", m["right"], h, eps)
    return 0.5 * (rms_norm(a, w[p + "left.out"], eps) + rms_norm(b, w[p + "right.out"], eps))


def feed_forward(w, p: str, h: torch.Tensor) -> torch.Tensor:
    return lin(w, p + "down", silu(lin(w, p + "gate", h)) * lin(w, p + "up", h))


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int]
            ) -> Tuple[torch.Tensor, List[torch.Tensor]]:
    """(logits [n, vocab], the residual stream after every layer)."""
    eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
    x = w["embed"].to(D)[torch.tensor(tokens)] * cfg["embedding"]["scale"]
    streams = []
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        mix = pooled_attention if layer["type"] == "attention" else side_by_side
        x = rms_norm(alpha * x + mix(w, p + "mix.", layer["mixer"], x, eps), w[p + "norm1"], eps)
        if layer.get("mlp"):
            x = rms_norm(alpha * x + feed_forward(w, p + "mlp.", x), w[p + "norm2"], eps)
        streams.append(x.clone())
    return lin(w, "head", rms_norm(x, w["final.norm"], eps)), streams
