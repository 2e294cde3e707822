"""The Dazilix design: config.json keys -> ModelConfig.

A Dazilix config names its design with ``"architecture": "Dazilix"`` and lists its layers one by one:

* ``vocab``, ``width``, ``norm.eps`` (of every norm of the model), ``embedding.scale`` (the embedded rows are multiplied
  by it);
* ``layers[i]``: ``type`` (the mixer: ``attention`` or ``gla``), ``mixer`` (its sizes and constants) and ``mlp``
  (``{"kind": "moe", ...}`` or null for none); layer i's tensors start with ``l<i>.``, its mixer's with ``l<i>.mix.``, its
  feed-forward's with ``l<i>.mlp.``. An RMS norm in front of each sublayer (``norm1`` / ``norm2``), one behind it (``norm1b``
  / ``norm2b``), and behind that a factor per channel (``ls1`` / ``ls2``);
* ``attention``: softmax attention inside chunks of ``mask.size`` positions (``heads``, ``kv_heads``, ``dim``, ``vdim``,
  ``scale``, used as given; ``rot`` with ``base`` and ``dims``: the pairs (i, i + dims / 2) among the first ``dims`` entries
  of every q and k head turn by p base^(-2i / dims)); the values are the keys as projected, so ``vdim`` is ``dim``; RMS
  norms over the whole q and the whole k projection; a one in the softmax's denominator;
* ``gla``: linear attention with a decay per key channel that the token chooses (``heads``, ``dim``, ``vdim``, ``tau``); the
  decay's input passes a narrow middle whose size is the tensors' (``a1`` / ``a2``), so it is read from the checkpoint
  when the weights are loaded;
* ``mlp``: ``router.experts`` / ``router.top`` (the chosen experts' weights are the softmax of their logits alone; the
  router has a bias), ``expert.ff``;
* ``loop`` (optional): layers ``start`` .. ``stop`` - 1 run ``times`` times in a row with one set of weights and a cache or
  state per pass; before every pass but the first the embedding output is added to the stream, then (before the first
  too) row t of ``loop.step`` [times, width].
"""
from __future__ import annotations

from typing import Any, List, Mapping

from .registry import register_architecture
from .schema import (ConfigError, LayerSpec, LinearAttentionSpec, ModelConfig, ModelNames, NormSpec, RopeSpec, RoutedMoeSpec,
                     ScheduleEntry, StreamVector, WideAttentionSpec)

MIXERS = ("attention", "gla")


def _need(m: Any, key: str, where: str):
    if not isinstance(m, Mapping) or key not in m or m[key] is None:
        raise ConfigError(f"config.json: {where} needs '{key}'")
    return m[key]


def _int(m: Any, key: str, where: str, least: int = 1) -> int:
    v = _need(m, key, where)
    if isinstance(v, bool) or not isinstance(v, (int, float)) or v != int(v) or int(v) < least:
        raise ConfigError(f"config.json: {where}.{key} must be an integer of at least {least}, got {v!r}")
    return int(v)


def _number(m: Any, key: str, where: str) -> float:
    v = _need(m, key, where)
    if isinstance(v, bool) or not isinstance(v, (int, float)):
        raise ConfigError(f"config.json: {where}.{key} must be a number, got {v!r}")
    return float(v)


def _attention(m: Any, w: str, eps: float, positions: List[RopeSpec]) -> WideAttentionSpec:
    heads, kv_heads = _int(m, "heads", w), _int(m, "kv_heads", w)
    if heads % kv_heads:
        raise ConfigError(f"config.json: {w}: {kv_heads} kv_heads do not divide {heads} heads")
    dim, vdim = _int(m, "dim", w), _int(m, "vdim", w)
    if vdim != dim:
        raise ConfigError(f"config.json: {w}: the values are the keys, so vdim={vdim} must be dim={dim}")
    rot = _need(m, "rot", w)
    dims = _int(rot, "dims", w + ".rot", least=2)
    if dims % 2 or dims > dim:
        raise ConfigError(f"config.json: {w}.rot.dims={dims} must be even and at most dim={dim}")
    rope = RopeSpec(rotary_dim=dims, theta=_number(rot, "base", w + ".rot"), pairing="half")
    if rope not in positions:
        positions.append(rope)
    return WideAttentionSpec(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=_number(m, "scale", w), eps=eps,
                             qk_norm="whole", position=positions.index(rope), bias=False, out_gate=False,
                             chunk=_int(_need(m, "mask", w), "size", w + ".mask"), tied_values=True, unit_sink=True)


def _gla(m: Any, w: str, eps: float) -> LinearAttentionSpec:
    dim, tau = _int(m, "dim", w), _number(m, "tau", w)
    if tau <= 0:
        raise ConfigError(f"config.json: {w}.tau must be positive, got {tau}")
    # the middle's size is the tensors' own: -1 = taken from the checkpoint at load
    return LinearAttentionSpec(heads=_int(m, "heads", w), dim=dim, vdim=_int(m, "vdim", w), decay=(), eps=eps,
                               k_scale=dim ** -0.5,  # of q in the design: (c q) . k = q . (c k), and the state is k's alone
                               norm="head_gain", gate_fn="silu", decay_per="channel", tau=tau, decay_rank=-1)


def _moe(mlp: Any, w: str) -> RoutedMoeSpec:
    kind = _need(mlp, "kind", w)
    if kind != "moe":
        raise ConfigError(f"config.json: {w}.kind '{kind}' is not a feed-forward of this design (moe is)")
    router, expert = _need(mlp, "router", w), _need(mlp, "expert", w)
    experts, top = _int(router, "experts", w + ".router"), _int(router, "top", w + ".router")
    if top > experts:
        raise ConfigError(f"config.json: {w}.router: top={top} of {experts} experts")
    return RoutedMoeSpec(experts=experts, top=top, hidden=_int(expert, "ff", w + ".expert"), correction=False, score="softmax",
                         normalize=True, router_bias=True)


def parse_dazilix(c: Mapping[str, Any], model_type: str, architecture: str) -> ModelConfig:
    vocab = _int(c, "vocab", "config")
    width = _int(c, "width", "config")
    eps = _number(_need(c, "norm", "config"), "eps", "norm")
    raw_layers = _need(c, "layers", "config")
    if not isinstance(raw_layers, (list, tuple)) or not raw_layers:
        raise ConfigError("config.json: layers must be a non-empty list")
    norm = NormSpec(eps=eps)
    positions: List[RopeSpec] = []
    layers = []
    for i, layer in enumerate(raw_layers):
        where = f"layers[{i}]"
        kind = _need(layer, "type", where)
        m = _need(layer, "mixer", where)
        if kind == "attention":
            mixer = _attention(m, where + ".mixer", eps, positions)
        elif kind == "gla":
            mixer = _gla(m, where + ".mixer", eps)
        else:
            raise ConfigError(f"config.json: {where}.type '{kind}' is not a mixer of this design ({', '.join(MIXERS)})")
        mlp = layer.get("mlp")
        ffn = _moe(mlp, where + ".mlp") if mlp is not None else None
        layers.append(LayerSpec(mixer=mixer, ffn=ffn, norm=norm, prefix=f"l{i}", arrangement="sandwich", norm_in_name="norm1",
                                norm_mixer_out_name="norm1b", norm_post_name="norm2", norm_ffn_out_name="norm2b",
                                mixer_scale_name="ls1", ffn_scale_name="ls2", name_ending="", mixer_prefix="mix"))
    n = len(layers)
    loop = c.get("loop")
    if loop is None:
        schedule = [ScheduleEntry(i) for i in range(n)]
        looped = ""
    else:
        start, stop, times = _int(loop, "start", "loop", 0), _int(loop, "stop", "loop", 0), _int(loop, "times", "loop", 0)
        if not start <= stop <= n:
            raise ConfigError(f"config.json: loop runs layers {start} .. {stop} - 1 of {n}")
        schedule = [ScheduleEntry(i) for i in range(start)]
        for t in range(times):
            schedule += [ScheduleEntry(i, add_before=StreamVector("loop.step", times, t) if i == start else None,
                                       add_embedding=i == start and t > 0) for i in range(start, stop)]
        schedule += [ScheduleEntry(i) for i in range(stop, n)]
        looped = f" loop={start}..{stop - 1}x{times}"
    kinds = [l["type"] for l in raw_layers]
    description = (f"{architecture} width={width} layers={n} runs={len(schedule)} vocab={vocab} "
                   + " ".join(f"{k}={kinds.count(k)}" for k in MIXERS) + looped)
    longest = c.get("max_positions")
    embedding = c.get("embedding")
    return ModelConfig(
        architecture=architecture, model_type=model_type, hidden=width, vocab=vocab, final_norm=norm, layers=tuple(layers),
        positions=tuple(positions), schedule=tuple(schedule), tie_embeddings=False,
        max_positions=int(longest) if isinstance(longest, int) and longest > 0 else 4096,
        embed_scale=_number(embedding, "scale", "embedding") if embedding is not None else 1.0, description=description,
        names=ModelNames(embed="embed", final_norm="final.norm", head="head"), raw=dict(c))


register_architecture("dazilix", "Dazilix", parse_dazilix, replace=True)
