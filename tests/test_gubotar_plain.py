"""Gubotar on the CPU: the parser, the pages and states a model asks for, pages given back where a chunk ends, the
engine's rotation table and the decays' powers against the plain formulas, the chunk plan, the random-weights mode, and
invariants of the plain implementation that its plausible misreadings fail."""
import json

import pytest
import torch

import gubotar_tiny as gt
from plain import gubotar_plain as P

F64 = torch.float64


def test_parser_reads_every_size_and_constant_from_the_config():
    from jllm_serve_amd.config import parse_config
    from jllm_serve_amd.config.schema import GatedMlpSpec, LinearAttentionSpec, ParallelMixerSpec, WideAttentionSpec
    c = parse_config(gt.G_A)
    assert c.architecture == "Gubotar" and c.hidden == 96 and c.vocab == 150 and len(c.layers) == 5 and c.tie_embeddings
    assert all(l.arrangement == "postnorm" and l.norm.kind == "rmsnorm" and l.norm.one_plus and l.norm.eps == 1e-6 for l in c.layers)
    assert c.final_norm.one_plus and c.final_norm.eps == 1e-6 and all(l.token_shift == "shift" for l in c.layers)
    p = c.layers[0].mixer
    assert isinstance(p, ParallelMixerSpec) and p.scales == (0.5, 0.5) and p.out_norms == ("left.out", "right.out") and p.out_eps == 1e-6
    left, right = p.branches
    assert isinstance(left, WideAttentionSpec) and (left.heads, left.kv_heads, left.dim, left.vdim, left.chunk, left.scale) == (6, 2, 12, 12, 7, 0.4)
    assert left.tied_values and left.head_temp and left.distance_bias and left.qk_norm == "head" and left.window == 0
    assert not left.bias and not left.out_gate and left.position is None and left.eps == 1e-6 and left.softcap == 0 and not left.sink
    assert isinstance(right, LinearAttentionSpec) and (right.heads, right.dim, right.vdim) == (3, 10, 14)
    assert right.decay == (0.5, 0.93, 0.998) and right.activation == "silu" and right.norm == "whole" and right.gate_fn == "sigmoid"
    assert right.position is None and right.k_scale == 1.0 and right.eps == 1e-6
    r = c.layers[1].mixer
    assert isinstance(r, LinearAttentionSpec) and (r.heads, r.dim, r.vdim, r.decay) == (2, 20, 12, (0.97, 1.0))
    assert r.activation is None and r.norm == "head" and r.gate_fn == "silu" and r.k_scale == pytest.approx(20 ** -0.5, rel=1e-12)
    rope = c.positions[r.position]
    assert (rope.rotary_dim, rope.theta, rope.pairing) == (8, 100.0, "half")
    assert c.positions[c.layers[2].mixer.position].theta == 40.0 and len(c.positions) == 2
    assert isinstance(c.layers[0].ffn, GatedMlpSpec) and c.layers[0].ffn.hidden == 56 and c.layers[0].ffn.activation == "silu"
    assert c.layers[2].ffn is None and c.layers[3].ffn is None
    assert [e.layer for e in c.schedule] == [0, 1, 2, 3, 4]


@pytest.mark.parametrize("change, text", [
    (lambda c: c["layers"][0].update(type="window"), "not a mixer of this design"),
    (lambda c: c["layers"][0]["mixer"].pop("right"), "needs 'right'"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=4), "do not divide"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(vdim=8), "values are the keys"),
    (lambda c: c["layers"][0]["mixer"]["left"].pop("mask"), "needs 'mask'"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(decay=[0.5, 0.6]), "one number per head"),
    (lambda c: c["layers"][1]["mixer"].update(decay=[0.5, 1.5]), "in 0..1"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=7), "even"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=22), "at most dim"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "not a feed-forward of this design"),
    (lambda c: c.pop("width"), "width"),
    (lambda c: c.pop("norm"), "norm"),
    (lambda c: c.update(layers=[]), "non-empty"),
])
def test_parser_refuses(change, text):
    from jllm_serve_amd.config import ConfigError, parse_config
    c = json.loads(json.dumps(gt.G_A))
    change(c)
    with pytest.raises(ConfigError, match=text):
        parse_config(c)


def test_pages_and_states_a_model_asks_for():
    from jllm_serve_amd.cache import CacheManager
    from jllm_serve_amd.config import parse_config
    from jllm_serve_amd.parts import DecoderModel
    model = DecoderModel(parse_config(gt.G_A), torch.float32, "cpu", 64)
    plans = model.cache_plans()
    assert [p.kv is not None for p in plans] == [True, False, False, True, True]
    assert [(r.name, r.shape) for r in plans[0].kv.rows] == [("k", (2, 12)), ("v", (2, 12))]
    assert [p.kv.chunk for p in plans if p.kv] == [7, 70, 33] and all(p.kv.window == 0 for p in plans if p.kv)
    # every run: the row before (token shift), then the recurrent matrices column by column
    assert [[s.shape for s in p.state] for p in plans] == [[(96,), (3, 14, 10)], [(96,), (2, 12, 20)], [(96,), (3, 22, 6)],
                                                           [(96,), (1, 9, 18)], [(96,), (5, 8, 8)]]
    assert all(s.dtype == torch.float32 for p in plans for s in p.state)
    cm = CacheManager(plans, 8, 256, 3, allocate=False, prefix_share=True)
    assert cm.tree is None and "chunks" in cm.sharing_refused
    names = {s.name: s.shape for s in model.weight_specs()}
    assert names["l0.mix.left.temp"] == (6,) and names["l0.mix.left.k.norm"] == (12,) and names["l0.mix.left.out"] == (96,)
    assert names["l0.mix.right.norm"] == (42,) and names["l1.mix.g"] == (24, 96) and names["l1.shift"] == (96,)
    assert not any(n.endswith("left.v") or n.endswith("left.g") for n in names)
    assert "l2.norm1" in names and "l2.norm2" not in names and not any(n.startswith("l2.mlp") for n in names)
    only = DecoderModel(parse_config(gt.G_C), torch.float32, "cpu", 64)
    assert all(p.kv is None and p.state is not None for p in only.cache_plans()), "a model without pages"


def test_pages_go_back_when_their_chunk_is_complete():
    from jllm_serve_amd.cache import CacheManager
    from jllm_serve_amd.cache.manager import CacheEntryPlan, CacheRow, PageSpec
    spec = PageSpec((CacheRow("k", (1, 2), 1),), chunk=10)
    cm = CacheManager([CacheEntryPlan(kv=spec)], 4, 64, 2, allocate=False)
    cm.open("a")
    held = []
    for n in (7, 2, 1, 1, 3, 8, 20):
        cm.begin_write("a", n)
        cm.commit("a", n)
        t = cm.table("a", 0)
        first = cm.length("a") // 10 * 10  # what the next position still reads starts here
        assert all((p >= 0) == ((b + 1) * 4 > first) for b, p in enumerate(t)), (cm.length("a"), t)
        held.append(sum(p >= 0 for p in t))
        cm.check()
    assert held[:3] == [2, 3, 1], "positions 0 .. 9 are complete: pages 0 and 1 go, the page that 10 lies in stays"
    with pytest.raises(ValueError, match="already given back"):
        cm.truncate("a", 25)
    cm.truncate("a", 41)
    cm.close("a")
    cm.check()
    assert cm.free_pages() == [16]
    with pytest.raises(ValueError, match="a window or chunks"):
        PageSpec((CacheRow("k", (1, 2), 1),), window=3, chunk=4)


def test_visible_blocks_bounds_what_any_row_reads():
    from jllm_serve_amd.kernels import ops
    for span in (1, 2, 63, 64, 65, 100, 128, 300):
        for p in range(0, 700, 7):
            first_window, first_chunk = max(0, p + 1 - span), p // span * span
            for first in (first_window, first_chunk):
                assert p // 64 - first // 64 + 1 <= ops.visible_blocks(p + 1, span)
            kept = min(5, first_window)
            blocks = {j // 64 for j in range(first_window, p + 1)} | {j // 64 for j in range(kept)}
            assert len(blocks) <= ops.visible_blocks(p + 1, span, 5)
    assert ops.visible_blocks(1000) == 16 and ops.visible_blocks(1000, 5000) == 16


def test_powers_and_chunk_plan():
    from jllm_serve_amd.engine.step import Segment
    from jllm_serve_amd.kernels import ops
    p = ops.decay_powers([0.0, 1.0, 0.9, 0.999], "cpu").double()
    assert p.shape == (4, 65) and p[0, 0] == 1 and float(p[0, 1:].abs().max()) == 0 and bool((p[1] == 1).all())
    for h, d in ((2, 0.9), (3, 0.999)):
        assert torch.allclose(p[h], torch.tensor([d ** n for n in range(65)], dtype=F64), rtol=1e-7)
    req, ch = ops.linear_chunk_plan([Segment("a", 0, 0, 1, 9, 0), Segment("b", 1, 1, 130, 0, 1), Segment("c", 2, 131, 64, 3, 2)])
    assert req == [0, 1, 0, 1, 130, 1, 131, 64, 4]
    assert ch == [0, 1, 1, 64, 65, 64, 129, 2, 131, 64]


def test_engine_rotation_table_is_the_plain_one():
    from jllm_serve_amd.config import parse_config
    from jllm_serve_amd.parts.rope import rope_table
    for cfg in (gt.G_A, gt.G_B, gt.G_C):
        c = parse_config(cfg)
        for layer, raw in zip(c.layers, cfg["layers"]):
            if raw["type"] != "retention":
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
    folder = write_random_model(str(tmp_path / "m"), gt.G_A, 5)
    w = gt.load_weights(folder)
    assert w["l0.mix.left.q"].shape == (72, 96) and w["l3.mix.left.k"].shape == (30, 96) and "head" not in w
    assert float(w["l0.norm1"].abs().max()) < 0.2, "stored around zero"
    logits = P.forward(gt.G_A, w, gt.prompt("GA", 9))
    assert logits.shape == (9, 150) and bool(torch.isfinite(logits).all())


# ------------------------------------------------------------------------------------------------ the plain implementation


def test_plain_norm_has_its_eps_inside_the_root_and_a_gain_of_one_plus_w():
    x = torch.tensor([[3.0, -4.0]], dtype=F64)
    w = torch.tensor([0.0, 1.0], dtype=F64)
    want = torch.tensor([[3.0, -8.0]], dtype=F64) / (12.5 + 0.5) ** 0.5
    assert torch.allclose(P.centred_norm(x, w, 0.5), want)


def test_plain_token_shift_uses_the_unshifted_row_before():
    h = torch.tensor([[1.0, 10.0], [2.0, 20.0], [4.0, 40.0]], dtype=F64)
    mu = torch.tensor([0.5, 1.0], dtype=F64)
    assert P.token_shift(h, mu).tolist() == [[0.5, 0.0], [1.5, 10.0], [3.0, 20.0]]


def test_plain_attention_sees_its_chunk_and_takes_the_distance_off():
    m = P.visible(9, 4)
    assert m[3].tolist() == [True] * 4 + [False] * 5 and m[4].tolist() == [False] * 4 + [True] + [False] * 4
    assert m[8].tolist() == [False] * 8 + [True]
    assert P.slopes(4).tolist() == [2.0 ** -2, 2.0 ** -4, 2.0 ** -6, 2.0 ** -8]
    assert P.slopes(3)[0] == pytest.approx(2 ** (-8 / 3))
    q = torch.zeros(3, 2, 2, dtype=F64)  # equal scores: only the distance decides
    k = torch.zeros(3, 1, 2, dtype=F64)
    v = torch.eye(3, dtype=F64)[:, None, :]
    o = P.attend(q, k, v, 1.0, torch.ones(2, dtype=F64), torch.tensor([0.7, 0.0], dtype=F64), P.visible(3, 8))
    e = torch.exp(-0.7 * torch.tensor([2.0, 1.0, 0.0], dtype=F64))
    assert torch.allclose(o[2, 0], e / e.sum()) and torch.allclose(o[2, 1], torch.full((3,), 1 / 3, dtype=F64))


def test_plain_values_are_the_unnormed_keys():
    m = {"heads": 1, "kv_heads": 1, "dim": 2, "vdim": 2, "scale": 1.0, "mask": {"size": 1}}
    eye = torch.eye(2, dtype=F64)
    w = {"q": eye, "k": eye * 3, "o": eye, "q.norm": torch.ones(2, dtype=F64), "k.norm": torch.full((2,), 7.0, dtype=F64), "temp": torch.ones(1, dtype=F64)}
    h = torch.tensor([[1.0, 2.0], [-3.0, 0.5]], dtype=F64)  # chunks of one: every row returns its own value
    assert torch.allclose(P.chunk_attention(h, m, w, 1e-6), 3 * h)


def test_plain_memory_is_the_decayed_sum_and_reads_its_own_write():
    torch.manual_seed(1)
    q, k, v = torch.randn(7, 2, 3, dtype=F64), torch.randn(7, 2, 3, dtype=F64), torch.randn(7, 2, 4, dtype=F64)
    d = [0.5, 0.9]
    o, S = P.decayed_memory(q, k, v, d)
    for t in range(7):
        for h in range(2):
            want = sum(d[h] ** (t - s) * (q[t, h] @ k[s, h]) * v[s, h] for s in range(t + 1))
            assert torch.allclose(o[t, h], want)
    o1, S1 = P.decayed_memory(q[:3], k[:3], v[:3], d)
    o2, S2 = P.decayed_memory(q[3:], k[3:], v[3:], d, S1)
    assert torch.allclose(torch.cat([o1, o2]), o) and torch.allclose(S2, S)


def test_plain_rotation_is_relative_and_leaves_the_tail():
    torch.manual_seed(2)
    q, k = torch.randn(1, 1, 10, dtype=F64), torch.randn(1, 1, 10, dtype=F64)

    def score(pq, pk):
        return float((P.rotate_half(q, torch.tensor([pq]), 6, 50.0) * P.rotate_half(k, torch.tensor([pk]), 6, 50.0)).sum())
    assert score(9, 4) == pytest.approx(score(25, 20), abs=1e-12) and abs(score(9, 4) - score(9, 5)) > 1e-3
    r = P.rotate_half(q, torch.tensor([7]), 6, 50.0)
    assert torch.equal(r[..., 6:], q[..., 6:]) and not torch.allclose(r[..., :6], q[..., :6])
    c, s = torch.cos(torch.tensor(7.0, dtype=F64)), torch.sin(torch.tensor(7.0, dtype=F64))
    assert r[0, 0, 0] == pytest.approx(float(q[0, 0, 0] * c - q[0, 0, 3] * s)) and r[0, 0, 3] == pytest.approx(float(q[0, 0, 3] * c + q[0, 0, 0] * s))


@pytest.mark.parametrize("name", sorted(gt.CONFIGS))
def test_plain_logits_depend_on_earlier_tokens_only_and_on_the_first(name, tmp_path):
    cfg, seed, _ = gt.CONFIGS[name]
    w = gt.load_weights(gt.write_model(str(tmp_path / "a"), cfg, seed))
    toks = gt.prompt(name, 20)
    a = P.forward(cfg, w, toks)
    b = P.forward(cfg, w, toks[:11] + [(t + 1) % cfg["vocab"] for t in toks[11:]])
    assert torch.allclose(a[:11], b[:11], atol=1e-12) and not torch.allclose(a[11:], b[11:], atol=1e-3)
    c = P.forward(cfg, w, [(toks[0] + 1) % cfg["vocab"]] + toks[1:])
    assert float((a[-1] - c[-1]).abs().max()) > 1e-4, "the recurrences carry something from the first token to the last"


@pytest.mark.parametrize("tensor, layer", [("mix.left.temp", 0), ("mix.left.out", 0), ("mix.right.norm", 0), ("shift", 1), ("norm1", 1),
                                           ("norm2", 1), ("mix.left.k.norm", 3), ("mix.g", 2)])
def test_every_small_tensor_moves_the_logits(tensor, layer, tmp_path):
    w = gt.load_weights(gt.write_model(str(tmp_path / "a"), gt.G_A, 51))
    toks = gt.prompt("GA", 24)
    base = P.forward(gt.G_A, w, toks)
    w[f"l{layer}.{tensor}"] = w[f"l{layer}.{tensor}"] + 0.5
    assert float((P.forward(gt.G_A, w, toks) - base).abs().max()) > 1e-2 * float(base.abs().max())
