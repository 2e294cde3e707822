"""A plain, slow Dazilix forward pass: whole sequences, no cache, one function per mechanism.

Dazilix is a decoder-only design with an RMS norm in front of and behind each sublayer and a factor per channel on what
a sublayer returns, x <- x + ls1 * norm1b(mixer(norm1 x)) and x <- x + ls2 * norm2b(ff(norm2 x)). Two mixers: a softmax
attention inside chunks of the sequence (its values are its keys as projected; q and k are normed over the whole
projection, then partly rotated; the denominator has a one of its own), and linear attention whose state decays by a
factor per key channel that the token chooses. The feed-forward is a mixture of experts whose weights are a softmax over
the chosen logits. A run of layers may be repeated; a pass adds its own vector to the stream, a further pass the
embedding output before that. This file shares no code with the engine. Everything is torch on the CPU in the dtype of
its inputs (tests use float64). The config is the raw config.json dict, read here independently of the engine's parser.

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


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


# ----------------------------------------------------------------------------------------------- softmax attention


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


def visible(T: int, chunk: int) -> torch.Tensor:
    """[T, T] bool: query i sees key j when j <= i and both lie in the same chunk of the sequence."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    return (j <= i) & (torch.div(i, chunk, rounding_mode="floor") == torch.div(j, chunk, rounding_mode="floor"))


def softmax_plus_one(s: torch.Tensor, mask: torch.Tensor) -> torch.Tensor:
    """Row by row exp(s_j) / (1 + sum_j exp(s_j)) over the visible entries, 0 elsewhere."""
    s = s.masked_fill(~mask, float("-inf"))
    top = torch.clamp(s.amax(dim=-1, keepdim=True), min=0.0)
    e = torch.exp(s - top)
    return e / (torch.exp(-top) + e.sum(dim=-1, keepdim=True))


def attend(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, mask: torch.Tensor) -> torch.Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, dv]; query head h reads key/value head h // (H / G)."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        sc = torch.einsum("id,jd->ij", q[:, h], k[:, g]) * scale
        out[:, h] = softmax_plus_one(sc, mask) @ v[:, g]
    return out


def chunk_attention(h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor], positions: torch.Tensor, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    raw = linear(h, w["k"])
    q = (rms(linear(h, w["q"]), eps) * w["q.norm"]).view(T, H, d)
    k = (rms(raw, eps) * w["k.norm"]).view(T, G, d)
    rot = m["rot"]
    q, k = rotate_half(q, positions, rot["dims"], rot["base"]), rotate_half(k, positions, rot["dims"], rot["base"])
    o = attend(q, k, raw.view(T, G, d), m["scale"], visible(T, m["mask"]["size"]))
    return linear(o.reshape(T, H * d), w["o"])


# ----------------------------------------------------------------------------------------------- linear attention


def channel_memory(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, alpha: torch.Tensor,
                   start: Optional[torch.Tensor] = None) -> Tuple[torch.Tensor, torch.Tensor]:
    """q, k, alpha [T, H, dk], v [T, H, dv]: token by token row c of S_h shrinks by alpha_c, then S_h += k v^T and
    o = S_h^T q. Returns (o [T, H, dv], the last S [H, dk, dv])."""
    T, H, dk = q.shape
    S = torch.zeros(H, dk, v.shape[2], dtype=q.dtype) if start is None else start.clone()
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for t in range(T):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = torch.einsum("hkv,hk->hv", S, q[t])
    return out, S


def channel_decay(z: torch.Tensor, tau: float) -> torch.Tensor:
    """sigmoid(z)^(1 / tau)"""
    return torch.exp(torch.nn.functional.logsigmoid(z) / tau)


def gated_linear_attention(h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor], eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    q, k = linear(h, w["q"]).view(T, H, d) * d ** -0.5, linear(h, w["k"]).view(T, H, d)
    v = linear(h, w["v"]).view(T, H, dv)
    alpha = channel_decay(linear(linear(h, w["a1"]), w["a2"]) + w["a2.b"], m["tau"]).view(T, H, d)
    o, _ = channel_memory(q, k, v, alpha)
    o = (rms(o, eps) * w["norm"]).reshape(T, H * dv) * silu(linear(h, w["g"]))
    return linear(o, w["o"])


# ----------------------------------------------------------------------------------------------- experts


def choose(z: torch.Tensor, top: int) -> Tuple[torch.Tensor, torch.Tensor]:
    """The ``top`` largest logits of every row and the softmax over those alone: (experts, weights) [T, top]."""
    best = torch.topk(z, top, dim=-1)
    return best.indices, torch.softmax(best.values, dim=-1)


def experts(h: torch.Tensor, mlp: dict, w: Dict[str, torch.Tensor]) -> torch.Tensor:
    which, weight = choose(linear(h, w["router"]) + w["router.b"], mlp["router"]["top"])
    out = torch.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        rows, place = (which == e).nonzero(as_tuple=True)
        if rows.numel() == 0:
            continue
        x = h[rows]
        y = linear(silu(linear(x, w[f"e{e}.gate"])) * linear(x, w[f"e{e}.up"]), w[f"e{e}.down"])
        out[rows] += y * weight[rows, place][:, None]
    return out


# ----------------------------------------------------------------------------------------------- layers


def mix(h: torch.Tensor, layer: dict, w: Dict[str, torch.Tensor], positions: torch.Tensor, eps: float) -> torch.Tensor:
    if layer["type"] == "attention":
        return chunk_attention(h, layer["mixer"], w, positions, eps)
    if layer["type"] == "gla":
        return gated_linear_attention(h, layer["mixer"], w, eps)
    raise ValueError(f"unknown mixer '{layer['type']}'")


def sub(weights: Dict[str, torch.Tensor], prefix: str) -> Dict[str, torch.Tensor]:
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def runs(cfg: dict) -> List[Tuple[int, Optional[int]]]:
    """The layers in the order they run, each with the number of the pass that starts with it (or None)."""
    n = len(cfg["layers"])
    loop = cfg.get("loop") or {"start": n, "stop": n, "times": 0}
    out: List[Tuple[int, Optional[int]]] = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        out += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return out + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg: dict, weights: Dict[str, torch.Tensor], tokens: List[int], watch=None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence from position 0. ``watch(run, x)`` gets the stream after every layer run."""
    positions = torch.arange(len(tokens))
    eps = float(cfg["norm"]["eps"])
    x0 = weights["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]
    x = x0
    for r, (i, begins) in enumerate(runs(cfg)):
        p = f"l{i}."
        layer = cfg["layers"][i]
        if begins is not None:
            if begins > 0:
                x = x + x0
            x = x + weights["loop.step"][begins]
        y = mix(rms(x, eps) * weights[p + "norm1"], layer, sub(weights, p + "mix."), positions, eps)
        x = x + rms(y, eps) * weights[p + "norm1b"] * weights[p + "ls1"]
        if layer.get("mlp"):
            y = experts(rms(x, eps) * weights[p + "norm2"], layer["mlp"], sub(weights, p + "mlp."))
            x = x + rms(y, eps) * weights[p + "norm2b"] * weights[p + "ls2"]
        if watch is not None:
            watch(r, x)
    return linear(rms(x, eps) * weights["final.norm"], weights["head"])


def generate(cfg: dict, weights: Dict[str, torch.Tensor], tokens: List[int], n: int) -> List[int]:
    """Greedy continuation of ``n`` tokens, the whole sequence computed anew for each."""
    seq = list(tokens)
    for _ in range(n):
        seq.append(int(torch.argmax(forward(cfg, weights, seq)[-1])))
    return seq[len(tokens):]
