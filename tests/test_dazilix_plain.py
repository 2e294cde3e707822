"""Dazilix on the CPU: the parser, the schedule of passes, the pages and states a model asks for, the engine's rotation
table against the plain formula, the random-weights mode, and invariants of the plain implementation that its plausible
misreadings fail."""
import json
import math

import pytest
import torch

import dazilix_tiny as dt
from plain import dazilix_plain as P

F64 = torch.float64


def test_parser_reads_every_size_and_constant_from_the_config():
    from jllm_serve_amd.config import parse_config
    from jllm_serve_amd.config.schema import LinearAttentionSpec, RoutedMoeSpec, WideAttentionSpec
    c = parse_config(dt.D_A)
    assert c.architecture == "Dazilix" and c.hidden == 90 and c.vocab == 131 and len(c.layers) == 5
    assert not c.tie_embeddings and c.embed_scale == 3.5 and c.final_norm.eps == 1e-6 and not c.final_norm.one_plus
    for l in c.layers:
        assert l.arrangement == "sandwich" and l.norm.kind == "rmsnorm" and l.norm.eps == 1e-6 and not l.norm.one_plus
        assert (l.norm_in_name, l.norm_mixer_out_name, l.norm_post_name, l.norm_ffn_out_name) == ("norm1", "norm1b", "norm2", "norm2b")
        assert (l.mixer_scale_name, l.ffn_scale_name) == ("ls1", "ls2")
    a = c.layers[1].mixer
    assert isinstance(a, WideAttentionSpec) and (a.heads, a.kv_heads, a.dim, a.vdim, a.chunk, a.scale) == (6, 2, 14, 14, 7, 0.3)
    assert a.tied_values and a.unit_sink and not a.sink and a.qk_norm == "whole" and a.eps == 1e-6 and a.window == 0
    assert not a.bias and not a.out_gate and not a.head_temp and not a.distance_bias and a.softcap == 0
    ropes = [c.positions[l.mixer.position] for l in (c.layers[1], c.layers[3], c.layers[4])]
    assert [(r.rotary_dim, r.theta, r.pairing) for r in ropes] == [(6, 60.0, "half"), (10, 700.0, "half"), (2, 10.0, "half")]
    g = c.layers[2].mixer
    assert isinstance(g, LinearAttentionSpec) and (g.heads, g.dim, g.vdim, g.tau) == (2, 21, 6, 0.5)
    assert g.decay_per == "channel" and g.decay == () and g.decay_rank == -1 and g.norm == "head_gain" and g.gate_fn == "silu"
    assert g.activation is None and g.position is None and g.k_scale == pytest.approx(21 ** -0.5, rel=1e-12) and g.eps == 1e-6
    m = c.layers[4].ffn
    assert isinstance(m, RoutedMoeSpec) and (m.experts, m.top, m.hidden, m.groups, m.scale) == (6, 5, 10, 1, 1.0)
    assert m.score == "softmax" and m.normalize and m.router_bias and not m.correction and m.activation == "silu" and m.shared is None
    assert c.layers[2].ffn is None and c.layers[3].ffn is None


def test_passes_of_a_loop():
    from jllm_serve_amd.config import parse_config
    c = parse_config(dt.D_A)
    assert [e.layer for e in c.schedule] == [0, 1, 2, 3, 1, 2, 3, 1, 2, 3, 4]
    starts = [i for i, e in enumerate(c.schedule) if e.add_before is not None]
    assert starts == [1, 4, 7] and [c.schedule[i].add_before.row for i in starts] == [0, 1, 2]
    assert all(c.schedule[i].add_before.rows == 3 and c.schedule[i].add_before.name == "loop.step" for i in starts)
    assert [i for i, e in enumerate(c.schedule) if e.add_embedding] == [4, 7], "the embedding output joins every pass but the first"
    assert all(e.cache_from is None for e in c.schedule), "a cache or state per pass"
    assert [e.layer for e in parse_config(dt.D_C).schedule] == [0, 1]
    d = parse_config(dt.D_D)
    assert [(e.layer, e.add_before is not None, e.add_embedding) for e in d.schedule] == [(0, False, False), (1, True, False)]
    assert P.runs(dt.D_A) == [(0, None), (1, 0), (2, None), (3, None), (1, 1), (2, None), (3, None), (1, 2), (2, None), (3, None), (4, None)]
    for cfg in (dt.D_A, dt.D_B, dt.D_C, dt.D_D):
        assert [i for i, _ in P.runs(cfg)] == [e.layer for e in parse_config(cfg).schedule]


@pytest.mark.parametrize("change, text", [
    (lambda c: c["layers"][0].update(type="window"), "not a mixer of this design"),
    (lambda c: c["layers"][0]["mixer"].pop("tau"), "needs 'tau'"),
    (lambda c: c["layers"][0]["mixer"].update(tau=0), "positive"),
    (lambda c: c["layers"][1]["mixer"].update(kv_heads=4), "do not divide"),
    (lambda c: c["layers"][1]["mixer"].update(vdim=8), "values are the keys"),
    (lambda c: c["layers"][1]["mixer"].pop("mask"), "needs 'mask'"),
    (lambda c: c["layers"][1]["mixer"].pop("scale"), "needs 'scale'"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=7), "even"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=16), "at most dim"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "not a feed-forward of this design"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=6), "top=6 of 5"),
    (lambda c: c["loop"].update(stop=6), "loop runs layers"),
    (lambda c: c.pop("width"), "width"),
    (lambda c: c.pop("norm"), "norm"),
    (lambda c: c.update(layers=[]), "non-empty"),
])
def test_parser_refuses(change, text):
    from jllm_serve_amd.config import ConfigError, parse_config
    c = json.loads(json.dumps(dt.D_A))
    change(c)
    with pytest.raises(ConfigError, match=text):
        parse_config(c)


def test_a_run_cannot_both_mix_and_add_the_embedding_output():
    import dataclasses
    from jllm_serve_amd.config import ConfigError, parse_config
    from jllm_serve_amd.config.schema import StreamMix
    c = parse_config(dt.D_A)
    bad = dataclasses.replace(c.schedule[4], mix_before=StreamMix("loop.in"))
    with pytest.raises(ConfigError, match="both mixes"):
        dataclasses.replace(c, schedule=c.schedule[:4] + (bad,) + c.schedule[5:])


def test_pages_states_and_tensors_a_model_asks_for():
    from jllm_serve_amd.cache import CacheManager
    from jllm_serve_amd.config import parse_config
    from jllm_serve_amd.parts import DecoderModel
    model = DecoderModel(parse_config(dt.D_A), torch.float32, "cpu", 64)
    plans = model.cache_plans()
    assert [p.kv is not None for p in plans] == [False, True, False, True, True, False, True, True, False, True, True]
    assert [(r.name, r.shape) for r in plans[1].kv.rows] == [("k", (2, 14)), ("v", (2, 14))]
    assert [p.kv.chunk for p in plans if p.kv] == [7, 70, 7, 70, 7, 70, 33] and all(p.kv.window == 0 for p in plans if p.kv)
    assert plans[0].state.shape == (3, 14, 10) and plans[2].state.shape == plans[5].state.shape == (2, 6, 21)
    assert all(p.state is None or p.state.dtype == torch.float32 for p in plans)
    cm = CacheManager(plans, 8, 256, 3, allocate=False, prefix_share=True)
    assert cm.tree is None, "a recurrent state cannot be shared by prefix"
    specs = {s.name: s for s in model.weight_specs() if not s.optional}
    names = {n: s.shape for n, s in specs.items()}
    assert names["l1.mix.q.norm"] == (84,) and names["l1.mix.k.norm"] == (28,) and names["l1.ls1"] == (90,) and names["l1.ls2"] == (90,)
    assert names["l0.mix.norm"] == (14,) and names["l0.mix.a1"] == (-1, 90) and names["l0.mix.a2"] == (30, -1) and names["l0.mix.a2.b"] == (30,)
    assert names["l0.mlp.router"] == (5, 90) and names["l0.mlp.router.b"] == (5,) and names["loop.step"] == (3, 90) and names["head"] == (131, 90)
    assert not any(n.endswith(("mix.sink", "mix.temp")) for n in names) and "l1.mix.v" not in names and "l1.mix.g" not in names
    assert "l2.ls1" in names and not any(n in names for n in ("l2.norm2", "l2.norm2b", "l2.ls2")) and not any(n.startswith("l2.mlp") for n in names)
    only = DecoderModel(parse_config(dt.D_C), torch.float32, "cpu", 64)
    assert all(p.kv is None and p.state is not None for p in only.cache_plans()), "a model without pages"


@pytest.mark.parametrize("middle", [1, 5, 32, 40])
def test_the_decays_middle_is_the_checkpoints_and_is_filled_up(middle, tmp_path):
    from jllm_serve_amd.config import parse_config
    from jllm_serve_amd.kernels import ops
    from jllm_serve_amd.parts import DecoderModel
    from jllm_serve_amd.weights.loader import TensorSource
    w = dt.load_weights(dt.write_model(str(tmp_path / "m"), dt.D_C, 3, middle=middle))
    model = DecoderModel(parse_config(dt.D_C), torch.float32, "cpu", 64)
    model.load(TensorSource({k: v.float() for k, v in w.items()}))
    m = model.layers[0].mixer
    full = -(-middle // ops.LINEAR_MIDDLE) * ops.LINEAR_MIDDLE
    assert m.decay_rank == middle and m.w_decay_up.shape == (30, full) and m.w_in.shape[0] >= m.decay_at + full
    assert torch.equal(m.w_decay_up[:, :middle].double(), w["l0.mix.a2"]) and float(m.w_decay_up[:, middle:].abs().sum()) == 0
    assert torch.equal(m.w_in[m.decay_at:m.decay_at + middle].double(), w["l0.mix.a1"]) and float(m.w_in[m.decay_at + middle:].abs().sum()) == 0
    # the factors per channel ride on the output norms
    assert torch.allclose(model.layers[0].norm_mixer_out.gain32.double(), w["l0.norm1b"] * w["l0.ls1"], rtol=1e-6)
    bad = {k: v.float() for k, v in w.items()}
    bad["l0.mix.a2"] = torch.zeros(30, middle + 1)
    with pytest.raises(ValueError, match="disagree"):
        model.load(TensorSource(bad))


def test_engine_rotation_table_is_the_plain_one():
    from jllm_serve_amd.config import parse_config
    from jllm_serve_amd.parts.rope import rope_table
    for cfg in (dt.D_A, dt.D_B, dt.D_D):
        c = parse_config(cfg)
        for layer, raw in zip(c.layers, cfg["layers"]):
            if raw["type"] != "attention":
                continue
            rot = raw["mixer"]["rot"]
            cos, sin = rope_table(c.positions[layer.mixer.position], 70)
            x = torch.zeros(70, 1, rot["dims"], dtype=F64)
            x[..., 0:rot["dims"] // 2] = 1.0
            r = P.rotate_half(x, torch.arange(70), rot["dims"], rot["base"])[:, 0]
            assert torch.allclose(torch.from_numpy(cos).double(), r[:, :rot["dims"] // 2], atol=1e-6)
            assert torch.allclose(torch.from_numpy(sin).double(), r[:, rot["dims"] // 2:], atol=1e-6)


def test_random_weights_mode_writes_what_the_model_loads(tmp_path):
    from jllm_serve_amd.weights import write_random_model
    folder = write_random_model(str(tmp_path / "m"), dt.D_A, 5)
    w = dt.load_weights(folder)
    assert w["l1.mix.q"].shape == (84, 90) and w["l4.mix.k"].shape == (18, 90) and w["head"].shape == (131, 90)
    assert "l2.norm2" not in w and "l1.mix.v" not in w
    logits = P.forward(dt.D_A, w, dt.prompt("DA", 9))
    assert logits.shape == (9, 131) and bool(torch.isfinite(logits).all())


# ------------------------------------------------------------------------------------------------ the plain implementation


def test_plain_norm_has_its_eps_inside_the_root():
    x = torch.tensor([[3.0, -4.0]], dtype=F64)
    assert torch.allclose(P.rms(x, 0.5), torch.tensor([[3.0, -4.0]], dtype=F64) / (12.5 + 0.5) ** 0.5)


def test_plain_softmax_has_a_one_in_its_denominator():
    s = torch.tensor([[0.0, 1.0, 50.0], [-700.0, -800.0, 0.0], [900.0, 899.0, 0.0]], dtype=F64)
    mask = torch.tensor([[True, True, False], [True, True, False], [True, True, False]])
    p = P.softmax_plus_one(s, mask)
    e = math.e
    assert torch.allclose(p[0], torch.tensor([1 / (2 + e), e / (2 + e), 0.0], dtype=F64))
    assert float(p[1].sum()) < 1e-300, "scores far below the sink's: nothing is looked at"
    assert torch.allclose(p[2], torch.tensor([e / (1 + e), 1 / (1 + e), 0.0], dtype=F64))


def test_plain_attention_sees_its_chunk_and_its_values_are_the_projected_keys():
    m = P.visible(9, 4)
    assert m[3].tolist() == [True] * 4 + [False] * 5 and m[4].tolist() == [False] * 4 + [True] + [False] * 4
    eye = torch.eye(4, dtype=F64)
    mixer = {"heads": 2, "kv_heads": 2, "dim": 2, "vdim": 2, "scale": 0.7, "mask": {"size": 1}, "rot": {"base": 10.0, "dims": 2}}
    w = {"q": eye, "k": eye * 3, "o": eye, "q.norm": torch.ones(4, dtype=F64), "k.norm": torch.full((4,), 5.0, dtype=F64)}
    h = torch.tensor([[1.0, 2.0, -1.0, 0.5], [-3.0, 0.5, 2.0, 1.0]], dtype=F64)
    o = P.chunk_attention(h, mixer, w, torch.arange(2), 1e-6)
    for t in range(2):  # chunks of one: a row returns its own value times exp(s) / (1 + exp(s)), with q and k normed over all heads
        n = h[t] / torch.sqrt((h[t] ** 2).mean())
        for head in range(2):
            s = 0.7 * 5.0 * float((n[2 * head:2 * head + 2] ** 2).sum())
            assert torch.allclose(o[t, 2 * head:2 * head + 2], 3 * h[t, 2 * head:2 * head + 2] / (1 + math.exp(-s)), atol=1e-5)


def test_plain_memory_decays_by_key_channel_and_reads_its_own_write():
    torch.manual_seed(1)
    T, H, dk, dv = 7, 2, 3, 4
    q, k, v = torch.randn(T, H, dk, dtype=F64), torch.randn(T, H, dk, dtype=F64), torch.randn(T, H, dv, dtype=F64)
    a = torch.rand(T, H, dk, dtype=F64)
    o, S = P.channel_memory(q, k, v, a)
    for t in range(T):
        for h in range(H):
            want = torch.zeros(dv, dtype=F64)
            for s in range(t + 1):  # the decays of the tokens behind s, not of s itself
                want += float((q[t, h] * k[s, h] * a[s + 1:t + 1, h].prod(dim=0)).sum()) * v[s, h]
            assert torch.allclose(o[t, h], want)
    o1, S1 = P.channel_memory(q[:3], k[:3], v[:3], a[:3])
    o2, S2 = P.channel_memory(q[3:], k[3:], v[3:], a[3:], S1)
    assert torch.allclose(torch.cat([o1, o2]), o) and torch.allclose(S2, S)
    z = torch.tensor([-900.0, -1.0, 0.0, 40.0], dtype=F64)
    assert torch.allclose(P.channel_decay(z, 2.0), torch.tensor([0.0, (1 / (1 + math.e)) ** 0.5, 0.5 ** 0.5, 1.0], dtype=F64))


def test_plain_router_softmaxes_the_chosen_logits_alone():
    z = torch.tensor([[1.0, 3.0, 2.0, -5.0]], dtype=F64)
    which, weight = P.choose(z, 2)
    assert which.tolist() == [[1, 2]] and torch.allclose(weight, torch.tensor([[math.e, 1.0]], dtype=F64) / (1 + math.e))


def test_plain_rotation_is_relative_and_leaves_the_tail():
    torch.manual_seed(2)
    q, k = torch.randn(1, 1, 10, dtype=F64), torch.randn(1, 1, 10, dtype=F64)

    def score(pq, pk):
        return float((P.rotate_half(q, torch.tensor([pq]), 6, 50.0) * P.rotate_half(k, torch.tensor([pk]), 6, 50.0)).sum())
    assert score(9, 4) == pytest.approx(score(25, 20), abs=1e-12) and abs(score(9, 4) - score(9, 5)) > 1e-3
    r = P.rotate_half(q, torch.tensor([7]), 6, 50.0)
    assert torch.equal(r[..., 6:], q[..., 6:]) and not torch.allclose(r[..., :6], q[..., :6])


@pytest.mark.parametrize("name", sorted(dt.CONFIGS))
def test_plain_logits_depend_on_earlier_tokens_only_and_on_the_first(name, tmp_path):
    cfg, seed, _, middle = dt.CONFIGS[name]
    w = dt.load_weights(dt.write_model(str(tmp_path / "a"), cfg, seed, middle))
    toks = dt.prompt(name, 20)
    a = P.forward(cfg, w, toks)
    b = P.forward(cfg, w, toks[:11] + [(t + 1) % cfg["vocab"] for t in toks[11:]])
    assert torch.allclose(a[:11], b[:11], atol=1e-12) and not torch.allclose(a[11:], b[11:], atol=1e-3)
    c = P.forward(cfg, w, [(toks[0] + 1) % cfg["vocab"]] + toks[1:])
    assert float((a[-1] - c[-1]).abs().max()) > 1e-4, "something is carried from the first token to the last"


@pytest.mark.parametrize("tensor", ["l0.mix.norm", "l0.mix.a2.b", "l0.mix.a1", "l0.mix.g", "l4.mlp.router.b", "l0.norm1b", "l0.ls1", "l0.ls2", "l1.mix.q.norm",
                                    "l1.mix.k.norm", "l1.norm2b", "l3.ls1", "loop.step", "l4.norm2", "final.norm"])
def test_every_small_tensor_moves_the_logits(tensor, tmp_path):
    w = dt.load_weights(dt.write_model(str(tmp_path / "a"), dt.D_A, 61, 5))
    toks = dt.prompt("DA", 24)
    base = P.forward(dt.D_A, w, toks)
    g = torch.Generator().manual_seed(3)
    w[tensor] = w[tensor] + 3 * torch.randn(w[tensor].shape, generator=g, dtype=F64)
    assert float((P.forward(dt.D_A, w, toks) - base).abs().max()) > 1e-2 * float(base.abs().max())


def test_the_embedding_output_joins_later_passes(tmp_path):
    w = dt.load_weights(dt.write_model(str(tmp_path / "a"), dt.D_A, 61, 5))
    toks = dt.prompt("DA", 12)
    seen = []
    P.forward(dt.D_A, w, toks, watch=lambda r, x: seen.append(x.clone()))
    x0 = w["embed"][torch.tensor(toks)] * 3.5
    layer, p = dt.D_A["layers"][1], "l1."
    for before, row, x in ((seen[0], 0, seen[1]), (seen[3] + x0, 1, seen[4]), (seen[6] + x0, 2, seen[7])):
        s = before + w["loop.step"][row]
        y = P.mix(P.rms(s, 1e-6) * w[p + "norm1"], layer, P.sub(w, p + "mix."), torch.arange(12), 1e-6)
        s = s + w[p + "ls1"] * (P.rms(y, 1e-6) * w[p + "norm1b"])
        y = P.experts(P.rms(s, 1e-6) * w[p + "norm2"], layer["mlp"], P.sub(w, p + "mlp."))
        assert torch.allclose(x, s + w[p + "ls2"] * (P.rms(y, 1e-6) * w[p + "norm2b"]))
