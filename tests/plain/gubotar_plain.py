"""A plain, slow Gubotar forward pass: whole sequences, no cache, one function per mechanism.

Gubotar is a decoder-only design whose layers norm only what a sublayer returns, x <- x + norm1(mixer(shifted x)) and
x <- x + norm2(ff(x)), with an RMS norm whose stored weight w means a gain of 1 + w. What a mixer reads is mixed with
the previous token's row element by element. Two mixers: linear attention with a fixed decay per head (retention), and
two mixers side by side whose outputs are normed before they are averaged: a softmax attention inside chunks of the
sequence, whose values are its unnormed keys, with a number and a distance penalty per head on the scores, and linear
attention with a fixed decay and silu on q, k and v. The head is the embedding table. This file shares no code with
the engine. Everything is torch on the CPU in the dtype of its inputs (tests use float64). The config is the raw
config.json dict, read here independently of the engine's parser.

Notation: h is a sublayer's input [T, width]; W are stored [out, in] and applied as W h.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Tuple

import torch


def linear(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    return torch.einsum("tc,rc->tr", x, w)


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last axis, eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def centred_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """RMS norm with the gain 1 + w."""
    return rms(x, eps) * (1.0 + w)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def token_shift(h: torch.Tensor, mu: torch.Tensor) -> torch.Tensor:
    """Row t becomes h_t + mu (h_(t-1) - h_t), with the unchanged row before it and zeros before the first."""
    before = torch.cat([torch.zeros_like(h[:1]), h[:-1]], dim=0)
    return h + (before - h) * mu


# ----------------------------------------------------------------------------------------------- softmax attention


def slopes(heads: int) -> torch.Tensor:
    """Head h of H takes 2^(-8 (h + 1) / H) off a score per position of distance."""
    return torch.pow(torch.tensor(2.0, dtype=torch.float64), -8.0 * torch.arange(1, heads + 1, dtype=torch.float64) / heads)


def visible(T: int, chunk: int) -> torch.Tensor:
    """[T, T] bool: query i sees key j when j <= i and both lie in the same chunk of the sequence."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    return (j <= i) & (torch.div(i, chunk, rounding_mode="floor") == torch.div(j, chunk, rounding_mode="floor"))


def attend(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, temp: torch.Tensor, slope: torch.Tensor,
           mask: torch.Tensor) -> torch.Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, dv]; query head h reads key/value head h // (H / G). Scores (q . k) scale
    temp_h - slope_h (i - j), softmax over the visible keys."""
    T, H, _ = q.shape
    G = k.shape[1]
    dist = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).to(q.dtype)
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        sc = torch.einsum("id,jd->ij", q[:, h], k[:, g]) * scale * temp[h] - slope[h].to(q.dtype) * dist
        p = torch.softmax(sc.masked_fill(~mask, float("-inf")), dim=-1)
        out[:, h] = p @ v[:, g]
    return out


def chunk_attention(h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor], eps: float) -> torch.Tensor:
    """The left branch: q and k heads are RMS-normed with one gain vector each, the values are the k heads before
    that norm, no rotation."""
    T = h.shape[0]
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    q = linear(h, w["q"]).view(T, H, d)
    raw = linear(h, w["k"]).view(T, G, d)
    q = rms(q, eps) * w["q.norm"]
    k = rms(raw, eps) * w["k.norm"]
    o = attend(q, k, raw, m["scale"], w["temp"], slopes(H), visible(T, m["mask"]["size"]))
    return linear(o.reshape(T, H * d), w["o"])


# ----------------------------------------------------------------------------------------------- linear attention


def decayed_memory(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: List[float],
                   start: Optional[torch.Tensor] = None) -> Tuple[torch.Tensor, torch.Tensor]:
    """q, k [T, H, dk], v [T, H, dv]: token by token S_h <- decay_h S_h + k v^T, o = S_h^T q. Returns (o [T, H, dv],
    the last S [H, dk, dv])."""
    T, H, dk = q.shape
    S = torch.zeros(H, dk, v.shape[2], dtype=q.dtype) if start is None else start.clone()
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    d = torch.tensor(decay, dtype=q.dtype)[:, None, None]
    for t in range(T):
        S = d * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = torch.einsum("hkv,hk->hv", S, q[t])
    return out, S


def lightning(h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor], eps: float) -> torch.Tensor:
    """The right branch: silu on q, k and v; the concatenated heads are normed together with a weight, then gated."""
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    q, k = silu(linear(h, w["q"])).view(T, H, d), silu(linear(h, w["k"])).view(T, H, d)
    v = silu(linear(h, w["v"])).view(T, H, dv)
    o, _ = decayed_memory(q, k, v, m["decay"])
    o = rms(o.reshape(T, H * dv), eps) * w["norm"] * torch.sigmoid(linear(h, w["g"]))
    return linear(o, w["o"])


def rotate_half(x: torch.Tensor, positions: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """x [T, heads, n]: entry i and entry i + dims / 2 (i < dims / 2) turn by the angle p base^(-2i / dims); entries
    from dims on pass unchanged."""
    half = dims // 2
    f = torch.pow(torch.tensor(float(base), dtype=torch.float64), -2.0 * torch.arange(half, dtype=torch.float64) / dims)
    a = positions.to(torch.float64)[:, None] * f[None, :]
    c, s = torch.cos(a).to(x.dtype)[:, None, :], torch.sin(a).to(x.dtype)[:, None, :]
    out = x.clone()
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half] = u * c - v * s
    out[..., half:dims] = v * c + u * s
    return out


def retention(h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor], positions: torch.Tensor, eps: float) -> torch.Tensor:
    """q and k rotated, k times dim^(-1/2), every head's read-out divided by its root mean square, a silu gate."""
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    rot = m["rot"]
    q = rotate_half(linear(h, w["q"]).view(T, H, d), positions, rot["dims"], rot["base"])
    k = rotate_half(linear(h, w["k"]).view(T, H, d), positions, rot["dims"], rot["base"]) * d ** -0.5
    v = linear(h, w["v"]).view(T, H, dv)
    o, _ = decayed_memory(q, k, v, m["decay"])
    o = rms(o, eps).reshape(T, H * dv) * silu(linear(h, w["g"]))
    return linear(o, w["o"])


# ----------------------------------------------------------------------------------------------- layers


def side_by_side(h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor], eps: float) -> torch.Tensor:
    """Half the sum of the branches' outputs, each RMS-normed over the width with a weight of its own first."""
    left = chunk_attention(h, m["left"], sub(w, "left."), eps)
    right = lightning(h, m["right"], sub(w, "right."), eps)
    return 0.5 * (rms(left, eps) * w["left.out"] + rms(right, eps) * w["right.out"])


def gated_ff(h: torch.Tensor, w: Dict[str, torch.Tensor]) -> torch.Tensor:
    return linear(silu(linear(h, w["gate"])) * linear(h, w["up"]), w["down"])


def mix(h: torch.Tensor, layer: dict, w: Dict[str, torch.Tensor], positions: torch.Tensor, eps: float) -> torch.Tensor:
    if layer["type"] == "parallel":
        return side_by_side(h, layer["mixer"], w, eps)
    if layer["type"] == "retention":
        return retention(h, layer["mixer"], w, positions, eps)
    raise ValueError(f"unknown mixer '{layer['type']}'")


def sub(weights: Dict[str, torch.Tensor], prefix: str) -> Dict[str, torch.Tensor]:
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg: dict, weights: Dict[str, torch.Tensor], tokens: List[int], watch=None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence from position 0. ``watch(layer, x)`` gets the stream after every layer."""
    positions = torch.arange(len(tokens))
    eps = float(cfg["norm"]["eps"])
    x = weights["embed"][torch.tensor(tokens)]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = token_shift(x, weights[p + "shift"])
        x = x + centred_norm(mix(h, layer, sub(weights, p + "mix."), positions, eps), weights[p + "norm1"], eps)
        if layer.get("mlp"):
            x = x + centred_norm(gated_ff(x, sub(weights, p + "mlp.")), weights[p + "norm2"], eps)
        if watch is not None:
            watch(i, x)
    return linear(centred_norm(x, weights["final.norm"], eps), weights["embed"])


def generate(cfg: dict, weights: Dict[str, torch.Tensor], tokens: List[int], n: int) -> List[int]:
    """Greedy continuation of ``n`` tokens, the whole sequence computed anew for each."""
    seq = list(tokens)
    for _ in range(n):
        seq.append(int(torch.argmax(forward(cfg, weights, seq)[-1])))
    return seq[len(tokens):]
