"""The Gubotar design: config.json keys -> ModelConfig.

A Gubotar config names its design with ``"architecture": "Gubotar"`` and lists its layers one by one:

* ``vocab``, ``width``, ``norm.eps`` (of every norm of the model);
* ``layers[i]``: ``type`` (the mixer: ``parallel`` or ``retention``), ``mixer`` (its sizes and constants) and ``mlp``
  (``{"kind": "dense", "ff": ...}`` or null for none); layer i's tensors start with ``l<i>.``, its mixer's with
  ``l<i>.mix.``, its feed-forward's with ``l<i>.mlp.``. A layer norms what its sublayers return (``norm1`` / ``norm2``,
  weights stored around zero) and reads the stream itself; ``shift`` mixes what the mixer reads with the previous
  token's row;
* ``retention``: ``heads``, ``dim``, ``vdim``, ``decay`` (one number per head), ``rot`` (``base``, ``dims``: the pairs
  (i, i + dims / 2) among the first ``dims`` entries of every q and k head turn by p base^(-2i / dims));
* ``parallel``: ``left`` (softmax attention inside chunks of ``mask.size`` positions: ``heads``, ``kv_heads``, ``dim``,
  ``vdim``, ``scale``; its values are its keys, so ``vdim`` is ``dim``) and ``right`` (linear attention: ``heads``,
  ``dim``, ``vdim``, ``decay``), averaged after a norm each (``left.out`` / ``right.out``).

The head is the embedding table.
"""
from __future__ import annotations

from typing import Any, List, Mapping, Tuple

from .registry import register_architecture
from .schema import (ConfigError, GatedMlpNames, GatedMlpSpec, LayerSpec, LinearAttentionSpec, ModelConfig, ModelNames,
                     NormSpec, ParallelMixerSpec, RopeSpec, WideAttentionNames, WideAttentionSpec, default_schedule)

MIXERS = ("parallel", "retention")


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


def _decay(m: Any, heads: int, w: str) -> Tuple[float, ...]:
    d = _need(m, "decay", w)
    if not isinstance(d, (list, tuple)) or len(d) != heads or any(isinstance(v, bool) or not isinstance(v, (int, float)) for v in d):
        raise ConfigError(f"config.json: {w}.decay must list one number per head ({heads})")
    if any(not 0.0 <= float(v) <= 1.0 for v in d):
        raise ConfigError(f"config.json: {w}.decay must lie in 0..1, got {list(d)}")
    return tuple(float(v) for v in d)


def _retention(m: Any, w: str, eps: float, positions: List[RopeSpec]) -> LinearAttentionSpec:
    heads, dim = _int(m, "heads", w), _int(m, "dim", w)
    rot = _need(m, "rot", w)
    dims = _int(rot, "dims", w + ".rot", least=2)
    if dims % 2 or dims > dim:
        raise ConfigError(f"config.json: {w}.rot.dims={dims} must be even and at most dim={dim}")
    rope = RopeSpec(rotary_dim=dims, theta=_number(rot, "base", w + ".rot"), pairing="half")
    if rope not in positions:
        positions.append(rope)
    return LinearAttentionSpec(heads=heads, dim=dim, vdim=_int(m, "vdim", w), decay=_decay(m, heads, w), eps=eps,
                               position=positions.index(rope), k_scale=dim ** -0.5, norm="head", gate_fn="silu")


def _chunk_attention(m: Any, w: str, eps: float) -> WideAttentionSpec:
    heads, kv_heads = _int(m, "heads", w), _int(m, "kv_heads", w)
    if heads % kv_heads:
        raise ConfigError(f"config.json: {w}: {kv_heads} kv_heads do not divide {heads} heads")
    dim, vdim = _int(m, "dim", w), _int(m, "vdim", w)
    if vdim != dim:
        raise ConfigError(f"config.json: {w}: the values are the keys, so vdim={vdim} must be dim={dim}")
    return WideAttentionSpec(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=_number(m, "scale", w), eps=eps,
                             qk_norm="head", bias=False, out_gate=False, chunk=_int(_need(m, "mask", w), "size", w + ".mask"),
                             tied_values=True, head_temp=True, distance_bias=True, names=WideAttentionNames())


def _lightning(m: Any, w: str, eps: float) -> LinearAttentionSpec:
    heads = _int(m, "heads", w)
    return LinearAttentionSpec(heads=heads, dim=_int(m, "dim", w), vdim=_int(m, "vdim", w), decay=_decay(m, heads, w), eps=eps,
                               activation="silu", norm="whole", gate_fn="sigmoid")


def parse_gubotar(c: Mapping[str, Any], model_type: str, architecture: str) -> ModelConfig:
    vocab = _int(c, "vocab", "config")
    width = _int(c, "width", "config")
    eps = _number(_need(c, "norm", "config"), "eps", "norm")
    raw_layers = _need(c, "layers", "config")
    if not isinstance(raw_layers, (list, tuple)) or not raw_layers:
        raise ConfigError("config.json: layers must be a non-empty list")
    norm = NormSpec(eps=eps, one_plus=True)
    positions: List[RopeSpec] = []
    layers = []
    for i, layer in enumerate(raw_layers):
        where = f"layers[{i}]"
        kind = _need(layer, "type", where)
        m = _need(layer, "mixer", where)
        w = where + ".mixer"
        if kind == "retention":
            mixer = _retention(m, w, eps, positions)
        elif kind == "parallel":
            mixer = ParallelMixerSpec(branches=(_chunk_attention(_need(m, "left", w), w + ".left", eps),
                                                _lightning(_need(m, "right", w), w + ".right", eps)),
                                      scales=(0.5, 0.5), prefixes=("left", "right"), out_norms=("left.out", "right.out"),
                                      out_eps=eps)
        else:
            raise ConfigError(f"config.json: {where}.type '{kind}' is not a mixer of this design ({', '.join(MIXERS)})")
        mlp = layer.get("mlp")
        ffn = None
        if mlp is not None:
            if _need(mlp, "kind", where + ".mlp") != "dense":
                raise ConfigError(f"config.json: {where}.mlp.kind '{mlp['kind']}' is not a feed-forward of this design (dense is)")
            ffn = GatedMlpSpec(hidden=_int(mlp, "ff", where + ".mlp"), activation="silu",
                               names=GatedMlpNames(gate="mlp.gate", up="mlp.up", down="mlp.down", ending=""))
        layers.append(LayerSpec(mixer=mixer, ffn=ffn, norm=norm, prefix=f"l{i}", arrangement="postnorm",
                                norm_mixer_out_name="norm1", norm_ffn_out_name="norm2", name_ending="", mixer_prefix="mix",
                                token_shift="shift"))
    kinds = [l["type"] for l in raw_layers]
    description = f"{architecture} width={width} layers={len(layers)} vocab={vocab} " + " ".join(f"{k}={kinds.count(k)}" for k in MIXERS)
    longest = c.get("max_positions")
    return ModelConfig(
        architecture=architecture, model_type=model_type, hidden=width, vocab=vocab, final_norm=norm, layers=tuple(layers),
        positions=tuple(positions), schedule=default_schedule(len(layers)), tie_embeddings=True,
        max_positions=int(longest) if isinstance(longest, int) and longest > 0 else 4096, description=description,
        names=ModelNames(embed="embed", final_norm="final.norm", head="head"), raw=dict(c))


register_architecture("gubotar", "Gubotar", parse_gubotar, replace=True)
