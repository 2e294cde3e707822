"""Tiny Dazilix configurations for the tests, their weights, and helpers shared by the tests.

DA varies what a layer can vary: both mixers, key heads equal to the heads, a part of them and a single one, chunks
shorter than a page and longer than a 64-key block, a rotation over a part of the head and over all of it, value sizes on
both sides of the key size, a tau below, at and above 1, a single chosen expert, layers without a feed-forward, three
passes of a loop; none of its sizes suits the matrix-core kernels. DB has sizes in multiples of 16 / 64 (what those
kernels take), chunks that end on and off a 64-key block, key sizes in several of the chunked recurrence's instantiations
and a loop that starts at the first layer and ends with the last. DC has only the recurrent mixer (no pages at all), odd
sizes and no loop. DD has only the attention, one head on each side, chunks of a single position, one expert in all, and a
loop of a single pass.
"""
import json
import os
import random

import torch


def _att(heads, kv, dim, size, scale, dims, base):
    return "attention", {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": scale, "mask": {"size": size},
                         "rot": {"base": base, "dims": dims}}


def _gla(heads, dim, vdim, tau):
    return "gla", {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}


def _layer(kind_mixer, experts, top, ff):
    kind, mixer = kind_mixer
    mlp = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}} if experts else None
    return {"type": kind, "mixer": mixer, "mlp": mlp}


D_A = {
    "architecture": "Dazilix", "vocab": 131, "width": 90, "norm": {"eps": 1e-6}, "embedding": {"scale": 3.5},
    "layers": [
        _layer(_gla(3, 10, 14, 7.0), 5, 2, 22),
        _layer(_att(6, 2, 14, 7, 0.3, 6, 60.0), 7, 1, 18),
        _layer(_gla(2, 21, 6, 0.5), 0, 0, 0),
        _layer(_att(3, 3, 10, 70, 0.4, 10, 700.0), 0, 0, 0),
        _layer(_att(5, 1, 18, 33, 0.25, 2, 10.0), 6, 5, 10),
    ],
    "loop": {"start": 1, "stop": 4, "times": 3},
}

D_B = {
    "architecture": "Dazilix", "vocab": 288, "width": 128, "norm": {"eps": 1e-4}, "embedding": {"scale": 1.6},
    "layers": [
        _layer(_att(8, 2, 32, 100, 0.2, 16, 5000.0), 16, 3, 64),
        _layer(_gla(3, 64, 48, 4.0), 8, 2, 128),
        _layer(_gla(1, 160, 80, 1.0), 4, 4, 64),
        _layer(_att(4, 4, 48, 64, 0.15, 48, 1e4), 70, 6, 32),
    ],
    "loop": {"start": 0, "stop": 4, "times": 2},
}

D_C = {
    "architecture": "Dazilix", "vocab": 101, "width": 70, "norm": {"eps": 1e-5}, "embedding": {"scale": 1.0},
    "layers": [
        _layer(_gla(5, 6, 7, 2.0), 3, 2, 12),
        _layer(_gla(1, 33, 25, 30.0), 0, 0, 0),
    ],
}

D_D = {
    "architecture": "Dazilix", "vocab": 64, "width": 48, "norm": {"eps": 1e-5}, "embedding": {"scale": 2.0},
    "layers": [
        _layer(_att(1, 1, 16, 1, 0.5, 4, 100.0), 1, 1, 32),
        _layer(_att(1, 1, 24, 500, 0.35, 24, 300.0), 9, 9, 16),
    ],
    "loop": {"start": 1, "stop": 2, "times": 1},
}

# name -> (config, weight seed, page size, width of the decays' narrow middle)
CONFIGS = {"DA": (D_A, 61, 8, 5), "DB": (D_B, 62, 16, 24), "DC": (D_C, 63, 4, 1), "DD": (D_D, 64, 16, 16)}


def write_model(folder, cfg, seed, middle=16, std=0.09):
    """A model folder with random weights wide enough that every mechanism moves the logits: the embedding and the pass
    vectors N(0, 0.7), matrices N(0, std) (the attention's q and k gains 1.4 + N(0, 0.3), so that scores have a spread),
    norms 1 + N(0, 0.3), factors per channel 0.4 + N(0, 0.15), routers whose choice
    depends on the token but is seldom a close call (weights N(0, 0.08), biases N(0, 2)), and decays from nearly 0 to
    nearly 1 (their bias N(2, 2.5), their matrices N(0, 0.3))."""
    from jllm_serve_amd.weights.random_init import random_source
    from jllm_serve_amd.weights.safetensors_io import write_safetensors
    src = random_source(cfg, seed, std=std)
    tensors = {n: src.get(n) for n in src.names()}
    g = torch.Generator().manual_seed(seed + 77)

    def normal(shape, mean, sd):
        return (torch.randn(shape, generator=g) * sd + mean).to(torch.bfloat16)

    for n, t in tensors.items():
        last = n.rsplit(".", 1)[-1]
        if n in ("embed", "loop.step"):
            tensors[n] = normal(t.shape, 0.0, 0.7)
        elif n.endswith("a1"):
            tensors[n] = normal((middle, t.shape[1]), 0.0, 0.3)
        elif n.endswith("a2"):
            tensors[n] = normal((t.shape[0], middle), 0.0, 0.3)
        elif n.endswith("a2.b"):
            tensors[n] = normal(t.shape, 2.0, 2.5)
        elif n.endswith("router"):
            tensors[n] = normal(t.shape, 0.0, 0.08)
        elif n.endswith("router.b"):
            tensors[n] = normal(t.shape, 0.0, 2.0)
        elif n.endswith("q.norm") or n.endswith("k.norm"):
            tensors[n] = normal(t.shape, 1.4, 0.3)
        elif last in ("ls1", "ls2"):
            tensors[n] = normal(t.shape, 0.4, 0.15)
        elif last.startswith("norm"):
            tensors[n] = normal(t.shape, 1.0, 0.3)
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
    bits of mantissa can do to single rows (with routers whose choice it can turn); ``typical`` bounds the median over many
    rows, and the float32 run, which takes the same path through cache, state and batching, is held tightly."""
    m = float(ref.abs().max())
    return 1e-4 * m + 1e-6 if dtype == "float32" else 0.1 * m


def turned(dtype, rows):
    """How many of a whole model's rows may lie beyond ``tolerance``. A router's choice is a step function of its input: in
    bfloat16 the normed rows carry a rounding of a few parts in a thousand, which turns a close call between two experts
    here and there, and through states and caches the rows behind it."""
    return 0 if dtype == "float32" else max(1, rows // 25)


def typical(dtype):
    """What the median over many rows of |difference| / largest |logit| may be."""
    return 5e-6 if dtype == "float32" else 2e-2
