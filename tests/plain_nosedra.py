"""Nosedra in plain 64-bit arithmetic: one function per mechanism, whole sequences, no cache.

The oracle of the Nosedra tests. It shares no code with the engine: weights come as a dict
name -> tensor, the configuration as the dict that config.json holds. Notation: h is what a
sublayer reads; unit(x) = x / sqrt(mean(x^2) + eps).
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

D = torch.float64


def unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def offset_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """A norm whose weight is stored around zero."""
    return unit(x, eps) * (1.0 + w.to(D))


def lin(w: Dict[str, torch.Tensor], name: str, x: torch.Tensor, bias: bool = False) -> torch.Tensor:
    y = x @ w[name].to(D).T
    return y + w[name + ".b"].to(D) if bias else y


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def gelu(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def log_sigmoid(z: torch.Tensor) -> torch.Tensor:
    return -torch.log1p(torch.exp(-z.abs())) + torch.minimum(z, torch.zeros_like(z))


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.log1p(torch.exp(-z.abs())) + torch.maximum(z, torch.zeros_like(z))


# ---- attention ---------------------------------------------------------------------------------

def rotate(x: torch.Tensor, pos: torch.Tensor, rot: Optional[dict]) -> torch.Tensor:
    """x [n, heads, d]: pair (i, i + dims / 2) of every head turns by pos base^(-2i / dims) / factor."""
    dims = (rot or {}).get("dims", 0)
    if not dims:
        return x
    factor = (rot.get("scaling") or {}).get("factor", 1.0)
    half = dims // 2
    out = x.clone()
    for i in range(half):
        a = pos.to(D) * (rot["base"] ** (-2.0 * i / dims) / factor)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * c - v * s
        out[..., i + half] = v * c + u * s
    return out


def attend(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, sink: torch.Tensor) -> torch.Tensor:
    """Causal softmax attention of q [n, H, d] over k [n, G, d], v [n, G, dv]; head a's denominator
    has one more term, exp(sink[a]). Returns [n, H, dv]."""
    n, H = q.shape[:2]
    per = H // k.shape[1]
    seen = torch.arange(n)[None, :] <= torch.arange(n)[:, None]
    out = torch.zeros(n, H, v.shape[-1], dtype=D)
    for a in range(H):
        s = q[:, a] @ k[:, a // per].T * scale
        s = torch.where(seen, s, torch.full((), -math.inf, dtype=D))
        top = torch.maximum(s.max(-1, keepdim=True).values, sink[a].to(D))
        e = torch.exp(s - top)
        out[:, a] = e @ v[:, a // per] / (e.sum(-1, keepdim=True) + torch.exp(sink[a].to(D) - top))
    return out


def gated_attention(w, p: str, m: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    n, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    G = m.get("kv_heads", H)
    pos = torch.arange(n)
    q = unit(rotate(lin(w, p + "q", h).reshape(n, H, d), pos, m.get("rot")), eps)
    k = unit(rotate(lin(w, p + "k", h).reshape(n, G, d), pos, m.get("rot")), eps)
    v = lin(w, p + "v", h).reshape(n, G, dv)
    o = attend(q, k, v, m["scale"], w[p + "sink"]).reshape(n, -1)
    return lin(w, p + "o", o * torch.sigmoid(lin(w, p + "g", h)))


# ---- matrix memory with exponential gates ----------------------------------------------------------

def capped(z: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(z / cap)


def memory(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, write: torch.Tensor, keep: torch.Tensor,
           state=None):
    """q, k [n, H, d], v [n, H, dv]; write, keep [n, H]: the logarithms of the gates. Row by row,
    m' = max(keep + m, write), S' = exp(keep + m - m') S + exp(write - m') k v^T, z likewise with k
    alone, o = S'^T q / (max(|z' . q|, exp(-m')) + 1e-6). Returns (o [n, H, dv], (S, z, m))."""
    n, H, d = q.shape
    if state is None:
        state = (torch.zeros(H, d, v.shape[-1], dtype=D), torch.zeros(H, d, dtype=D), torch.zeros(H, dtype=D))
    S, z, m = state
    o = torch.zeros(n, H, v.shape[-1], dtype=D)
    for t in range(n):
        top = torch.maximum(keep[t] + m, write[t])
        a, b = torch.exp(keep[t] + m - top), torch.exp(write[t] - top)
        S = a[:, None, None] * S + b[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        z = a[:, None] * z + b[:, None] * k[t]
        m = top
        den = torch.maximum((z * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        o[t] = (S * q[t][:, :, None]).sum(1) / den[:, None]
    return o, (S, z, m)


def matrix_memory(w, p: str, m: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    n, H, d, dv, cap = h.shape[0], m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    q = lin(w, p + "q", h).reshape(n, H, d) * d ** -0.5
    k = lin(w, p + "k", h).reshape(n, H, d)
    v = lin(w, p + "v", h).reshape(n, H, dv)
    write = capped(lin(w, p + "i", h, bias=True), cap)
    keep = log_sigmoid(capped(lin(w, p + "f", h, bias=True), cap))
    o, _ = memory(q, k, v, write, keep)
    o = unit(o, eps).reshape(n, -1) * w[p + "norm"].to(D)
    return lin(w, p + "o", o * torch.sigmoid(lin(w, p + "g", h)))


def side_by_side(w, p: str, m: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    return m["left_scale"] * gated_attention(w, p + "left.", m["left"], h, eps) \
        + m["right_scale"] * matrix_memory(w, p + "right.", m["right"], h, eps)


# ---- state space with a decay per head and token ------------------------------------------------------

def causal_conv(x: torch.Tensor, taps: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """x [n, c], taps [c, n_taps] (the last one the row's own): per channel, zeros before the start."""
    n, nt = x.shape[0], taps.shape[1]
    padded = torch.cat([torch.zeros(nt - 1, x.shape[1], dtype=D), x])
    out = bias.to(D).expand(n, -1).clone()
    for j in range(nt):
        out += taps[:, j].to(D) * padded[j:j + n]
    return out


def state_space(x: torch.Tensor, B: torch.Tensor, C: torch.Tensor, dt: torch.Tensor, rate: torch.Tensor,
                state: Optional[torch.Tensor] = None):
    """x [n, H, dv], B, C [n, G, N], dt [n, H] (positive), rate [H] (positive): row by row
    S = exp(-rate dt) S + dt B x^T, y = S^T C with the group of the head. Returns (y, S)."""
    n, H, dv = x.shape
    per = H // B.shape[1]
    S = torch.zeros(H, B.shape[2], dv, dtype=D) if state is None else state
    y = torch.zeros(n, H, dv, dtype=D)
    for t in range(n):
        b, c = B[t].repeat_interleave(per, 0), C[t].repeat_interleave(per, 0)
        S = torch.exp(-rate * dt[t])[:, None, None] * S + dt[t][:, None, None] * b[:, :, None] * x[t][:, None, :]
        y[t] = (S * c[:, :, None]).sum(1)
    return y, S


def mamba2(w, p: str, m: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    n, H, dv, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner, gn = H * dv, G * N
    u = lin(w, p + "in", h)
    z, xbc, dt = u[:, :inner], u[:, inner:2 * inner + 2 * gn], u[:, 2 * inner + 2 * gn:]
    xbc = silu(causal_conv(xbc, w[p + "conv"], w[p + "conv.b"]))
    x = xbc[:, :inner].reshape(n, H, dv)
    B, C = xbc[:, inner:inner + gn].reshape(n, G, N), xbc[:, inner + gn:].reshape(n, G, N)
    dt = softplus(dt + w[p + "dt_bias"].to(D))
    y, _ = state_space(x, B, C, dt, torch.exp(w[p + "A_log"].to(D)))
    y = (y + w[p + "D"].to(D)[:, None] * x).reshape(n, inner) * silu(z)
    y = unit(y.reshape(n, m["norm_groups"], -1), eps).reshape(n, inner) * w[p + "norm"].to(D)
    return lin(w, p + "o", y)


# ---- the rest ------------------------------------------------------------------------------------------

def feed_forward(w, p: str, h: torch.Tensor) -> torch.Tensor:
    return lin(w, p + "down", gelu(lin(w, p + "gate", h, bias=True)) * lin(w, p + "up", h, bias=True), bias=True)


def token_side(w, p: str, layer: int, dim: int, tokens: torch.Tensor, x: torch.Tensor, eps: float) -> torch.Tensor:
    e = w["side.embed"].to(D)[tokens][:, layer * dim:(layer + 1) * dim]
    y = lin(w, p + "proj", gelu(lin(w, p + "gate", x)) * e)
    return unit(y, eps) * w[p + "norm"].to(D)


MIXERS = {"parallel": side_by_side, "mamba2": mamba2}


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int]
            ) -> Tuple[torch.Tensor, List[torch.Tensor]]:
    """(logits [n, vocab], the residual stream after every layer)."""
    eps, cap = cfg["norm"]["eps"], cfg.get("logit_softcap")
    ids = torch.tensor(tokens)
    x = w["embed"].to(D)[ids]
    streams = []
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + MIXERS[layer["type"]](w, p + "mix.", layer["mixer"], offset_norm(x, w[p + "norm1"], eps), eps)
        if layer.get("mlp"):
            x = x + feed_forward(w, p + "mlp.", offset_norm(x, w[p + "norm2"], eps))
        x = x + token_side(w, p + "side.", i, cfg["token_side"]["dim"], ids, x, eps)
        streams.append(x.clone())
    logits = lin(w, "head", offset_norm(x, w["final.norm"], eps))
    return (capped(logits, cap) if cap else logits), streams
