"""Tiny Gubotar configurations for the tests, their weights, and helpers shared by the tests.

GA varies what a layer can vary: both mixers, key heads equal to the heads, a part of them and a single one, chunks
shorter than a page and longer than a 64-key block, a rotation over a part of the head, value sizes on both sides of the
key size, decays up to 1, a layer without a feed-forward; none of its sizes suits the matrix-core kernels. (A decay of 0
is for the recurrence alone: behind the norm of a head that holds a single term only the sign of q . k is left, which
rounding decides where the two are orthogonal.) GB has sizes in multiples of 16 / 32 (what those kernels take), chunks
that end on and off a 64-key block and key sizes in all the chunked recurrence's instantiations. GC has only the
recurrent mixer (no pages at all) and odd sizes. GD has only the side-by-side mixer, one head on each side, and chunks of
a single position.
"""
import json
import os
import random

import torch


def _left(heads, kv, dim, size, scale):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": scale, "mask": {"size": size}}


def _right(heads, dim, vdim, decay):
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}


def _ret(heads, dim, vdim, decay, dims, base):
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay, "rot": {"base": base, "dims": dims}}


def _layer(kind, mixer, ff):
    return {"type": kind, "mixer": mixer, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def _par(left, right, ff):
    return _layer("parallel", {"left": left, "right": right}, ff)


G_A = {
    "architecture": "Gubotar", "vocab": 150, "width": 96, "norm": {"eps": 1e-6},
    "layers": [
        _par(_left(6, 2, 12, 7, 0.4), _right(3, 10, 14, [0.5, 0.93, 0.998]), 56),
        _layer("retention", _ret(2, 20, 12, [0.97, 1.0], 8, 100.0), 72),
        _layer("retention", _ret(3, 6, 22, [0.6, 0.9, 0.996], 6, 40.0), None),
        _par(_left(3, 3, 10, 70, 0.3), _right(1, 18, 9, [0.99]), None),
        _par(_left(4, 1, 16, 33, 0.25), _right(5, 8, 8, [0.2, 0.7, 0.95, 0.99, 0.9995]), 40),
    ],
}

G_B = {
    "architecture": "Gubotar", "vocab": 320, "width": 128, "norm": {"eps": 1e-5},
    "layers": [
        _layer("retention", _ret(3, 64, 48, [0.9, 0.99, 0.9995], 64, 10000.0), 192),
        _par(_left(8, 2, 32, 100, 0.2), _right(2, 128, 16, [0.98, 0.9]), 256),
        _par(_left(4, 4, 48, 64, 0.15), _right(3, 48, 80, [0.7, 0.96, 0.9992]), 160),
        _layer("retention", _ret(1, 160, 128, [0.995], 32, 500.0), 64),
    ],
}

G_C = {
    "architecture": "Gubotar", "vocab": 97, "width": 70, "norm": {"eps": 1e-4},
    "layers": [
        _layer("retention", _ret(5, 6, 7, [0.6, 0.9, 0.95, 0.99, 0.999], 4, 77.0), 33),
        _layer("retention", _ret(1, 14, 25, [0.985], 14, 3000.0), None),
    ],
}

G_D = {
    "architecture": "Gubotar", "vocab": 64, "width": 48, "norm": {"eps": 1e-5},
    "layers": [
        _par(_left(1, 1, 16, 1, 0.5), _right(1, 16, 32, [0.97]), 32),
        _par(_left(1, 1, 24, 500, 0.35), _right(2, 32, 16, [0.99, 0.8]), 48),
    ],
}

# name -> (config, weight seed, page size)
CONFIGS = {"GA": (G_A, 51, 8), "GB": (G_B, 52, 16), "GC": (G_C, 53, 4), "GD": (G_D, 54, 16)}


def write_model(folder, cfg, seed, std=0.09):
    """A model folder with random weights wide enough that every mechanism moves the logits: the embedding N(0, 0.7),
    matrices N(0, std) (the softmax attention's q and k gains 1.3 + N(0, 0.3), so that scores have a spread), the norms'
    weights around zero N(0, 0.2), the branches' gains 1 + N(0, 0.3), the heads' factors 1 + N(0, 0.4), the token shift
    N(0.4, 0.3)."""
    from jllm_serve_amd.weights.random_init import random_source
    from jllm_serve_amd.weights.safetensors_io import write_safetensors
    src = random_source(cfg, seed, std=std)
    tensors = {n: src.get(n) for n in src.names()}
    g = torch.Generator().manual_seed(seed + 77)

    def normal(shape, mean, sd):
        return (torch.randn(shape, generator=g) * sd + mean).to(torch.bfloat16)

    for n, t in tensors.items():
        last = n.rsplit(".", 1)[-1]
        if n == "embed":
            tensors[n] = normal(t.shape, 0.0, 0.7)
        elif last in ("norm1", "norm2") or n == "final.norm":
            tensors[n] = normal(t.shape, 0.0, 0.2)
        elif last == "norm" and ".left." in n:
            tensors[n] = normal(t.shape, 1.3, 0.3)
        elif last in ("out", "norm"):
            tensors[n] = normal(t.shape, 1.0, 0.3)
        elif last == "temp":
            tensors[n] = normal(t.shape, 1.0, 0.4)
        elif last == "shift":
            tensors[n] = normal(t.shape, 0.4, 0.3)
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_safetensors(os.path.join(folder, "model.safetensors"), tensors)
    return folder


def load_weights(folder):
    """The folder's tensors through the safetensors package (not the engine's reader): floats as float64."""
    from safetensors import safe_open
    out = {}
    with safe_open(os.path.join(folder, "model.safetensors"), framework="pt") as f:
        for k in f.keys():
            t = f.get_tensor(k)
            out[k] = t.to(torch.float64) if t.is_floating_point() else t
    return out


def prompt(name, length, seed=0):
    rng = random.Random(f"{name}/{length}/{seed}")
    v = CONFIGS[name][0]["vocab"]
    return [rng.randrange(v) for _ in range(length)]


def tolerance(dtype, ref):
    """Against float64, for one row of logits. The bfloat16 bound is what rounding of activations, keys and values to 8
    bits of mantissa can do to single rows (a key, a chunk's edge, a page or a state that is off moves a row by more);
    ``typical`` bounds the median over many rows, and the float32 run, which takes the same path through cache, state
    and batching, is held tightly."""
    m = float(ref.abs().max())
    return 5e-5 * m + 1e-6 if dtype == "float32" else 0.08 * m


def typical(dtype):
    """What the median over many rows of |difference| / largest |logit| may be."""
    return 5e-6 if dtype == "float32" else 2e-2
