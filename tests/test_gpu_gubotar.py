"""Gubotar on the GPU against the plain implementation (tests/plain/gubotar_plain.py): every mechanism alone (the norm
behind a sublayer with and without branches, the token shift across steps, both forms of the recurrence on memories that
are hundreds of tokens old, the attention with one key that decides at chunk and page edges), mixers through cache and
state, whole prompts against token-by-token decoding, portions down to two tokens, mixed batches on a pool that is used
again, the stream after every layer, long decoding through captured steps, greedy generation through the engine, and the
command line."""
import json
import os

import numpy as np
import pytest
import torch

import gubotar_tiny as gt
import replay
from plain import gubotar_plain as P

pytestmark = pytest.mark.gpu
DEV = "cuda"
F64 = torch.float64
NAMES = sorted(gt.CONFIGS)


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: gt.write_model(str(tmp_path_factory.mktemp("gubotar_" + name)), cfg, seed)
            for name, (cfg, seed, page) in gt.CONFIGS.items()}


@pytest.fixture(scope="module")
def built(folders):
    from jllm_serve_amd.engine import build_runner, load_model
    cache = {}

    def get(name, dtype, graphs=False):
        if (name, dtype, graphs) not in cache:
            model = load_model(folders[name], dtype, torch.device(DEV), max_positions=1024)
            cache[(name, dtype, graphs)] = (model, build_runner(model, page_size=gt.CONFIGS[name][2], pool_tokens=1024,
                                                                max_requests=4, graphs=graphs))
        return cache[(name, dtype, graphs)]
    return get


@pytest.fixture(scope="module")
def plain_logits(folders):
    memo = {}

    def get(name, tokens):
        key = (name, tuple(tokens))
        if key not in memo:
            memo[key] = P.forward(gt.CONFIGS[name][0], gt.load_weights(folders[name]), list(tokens))
        return memo[key]
    return get


def close(got, want, dtype, what=""):
    err = float((got.double().cpu() - want).abs().max())
    assert err <= gt.tolerance(dtype, want), f"{what}: {err} > {gt.tolerance(dtype, want)}"


def act_type(dtype):
    return torch.float32 if dtype == "float32" else torch.bfloat16


# ------------------------------------------------------------------------------------------------ norms and the shift


@pytest.mark.parametrize("width", [12, 70, 128, 1000, 1024, 1500, 2048, 3001, 4096, 8192])
def test_join_of_a_normed_output(width):
    """x += rms(a) g and x += rms(s1 rms(a) g1 + s2 rms(b) g2) g, with the new rows as they are, rounded, or shifted with
    the requests' states; rows with a stride of their own."""
    from jllm_serve_amd.kernels import ops
    torch.manual_seed(width)
    n, eps, beps = 5, 1e-3, 2e-3
    x = torch.randn(n, width) * 2
    a, b = torch.randn(n, width + 8) * 3, torch.randn(n, width + 8) * 0.2
    g, g1, g2, mu = (torch.randn(width) for _ in range(4))
    state = torch.randn(9, width)
    slots = torch.tensor([3, 0, 7, 8, 2], dtype=torch.int32)
    for two in (False, True):
        for act in (torch.float32, torch.bfloat16):
            aa, bb = a.to(act)[:, :width], b.to(act)[:, :width]
            t = aa.double()
            if two:
                t = 0.5 * P.rms(aa.double(), beps) * g1.double() + 0.25 * P.rms(bb.double(), beps) * g2.double()
            want = x.double() + P.rms(t, eps) * g.double()
            kw = dict(a2=bb.to(DEV), branch_gains=(g1.to(DEV), g2.to(DEV)), scales=(0.5, 0.25), branch_eps=beps) if two else {}
            for out in (None, torch.float32, torch.bfloat16):
                xd = x.to(DEV)
                got = ops.rms_seam(xd, aa.to(DEV), g.to(DEV), eps, out_dtype=out, **kw)
                assert torch.allclose(xd.cpu().double(), want, atol=3e-5, rtol=1e-5), (two, act, out)
                assert (got is None) if out is None else torch.equal(got, xd.to(out))
                if out is None:
                    continue
                xd, st = x.to(DEV), state.to(DEV)
                got = ops.rms_seam(xd, aa.to(DEV), g.to(DEV), eps, out_dtype=out, shift=mu.to(DEV), state=st, state_slots=slots.to(DEV), **kw)
                before = state[slots.long()].double()
                shifted = want + (before - want) * mu.double()
                assert torch.allclose(got.cpu().double(), shifted, atol=3e-5 if out == torch.float32 else 2e-2, rtol=1e-5 if out == torch.float32 else 1e-2)
                assert torch.equal(st.cpu()[slots.long()], xd.cpu()), "the state is the new row"
                others = [i for i in range(9) if i not in slots.tolist()]
                assert torch.equal(st.cpu()[others], state[others]), "a state row of no request was written"


@pytest.mark.parametrize("width", [10, 96, 1028, 3000])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_token_shift_across_steps(width, dtype):
    """Two requests in portions (down to single rows, both kinds of launch) and one that joins later, against the whole
    sequences; the first row of a sequence is shifted with zeros."""
    from jllm_serve_amd.kernels import ops
    torch.manual_seed(width)
    act = act_type(dtype)
    seqs = {"a": torch.randn(24, width), "b": torch.randn(24, width), "c": torch.randn(11, width)}
    mu = torch.rand(width)
    slot = {"a": 4, "b": 0, "c": 2}
    state = torch.zeros(6, width, device=DEV)
    at = {k: 0 for k in seqs}
    got = {k: [] for k in seqs}
    steps = [{"a": 5, "b": 2}, {"a": 1, "b": 1}, {"b": 3, "c": 1}, {"a": 2, "b": 1, "c": 7}, {"a": 1, "b": 1, "c": 1}, {"a": 15, "b": 16, "c": 2}]
    for st in steps:
        rows = torch.cat([seqs[k][at[k]:at[k] + n] for k, n in st.items()])
        req = torch.tensor([i for i, n in enumerate(st.values()) for _ in range(n)], dtype=torch.int32, device=DEV)
        slots = torch.tensor([slot[k] for k in st], dtype=torch.int32, device=DEV)
        out = ops.token_shift(rows.to(DEV), mu.to(DEV), state, req, slots, len(st), act).cpu()
        o = 0
        for k, n in st.items():
            got[k].append(out[o:o + n])
            at[k] += n
            o += n
    for k, h in seqs.items():
        assert at[k] == h.shape[0]
        want = P.token_shift(h.double(), mu.double())
        assert torch.allclose(torch.cat(got[k]).double(), want, atol=1e-6 if dtype == "float32" else 2e-2)
        assert torch.equal(state[slot[k]].cpu(), h[-1])
    assert float(state[[1, 3, 5]].abs().max()) == 0.0


@pytest.mark.parametrize("width", [12, 70, 1024, 600])
def test_norm_of_a_whole_row_in_front_of_its_gate(width):
    from jllm_serve_amd.kernels import ops
    torch.manual_seed(width)
    T, eps = 11, 1e-3
    y, z, wt = torch.randn(T, width) * 0.3, torch.randn(T, width + 5), torch.randn(width)
    for act in (torch.float32, torch.bfloat16):
        zz, ww = z.to(act)[:, 5:], wt.to(act)
        big = torch.zeros(T, width + 7, device=DEV)
        ops.gated_group_norm(y.to(DEV), zz.to(DEV), ww.to(DEV), eps, 1, torch.float32, gate_fn="sigmoid", gate_last=True,
                             out=big[:, 3:3 + width], out_mul=0.5)
        want = 0.5 * P.rms(y.double(), eps) * ww.double() * torch.sigmoid(zz.double())
        assert torch.allclose(big[:, 3:3 + width].cpu().double(), want, atol=1e-5)
        assert float(big[:, :3].abs().max()) == 0 and float(big[:, 3 + width:].abs().max()) == 0


# ------------------------------------------------------------------------------------------------ the recurrence


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H, dk, dv, rot, silu", [(3, 16, 16, 0, True), (3, 64, 48, 64, False), (4, 128, 128, 32, False), (3, 256, 256, 64, False),
                                                  (3, 48, 176, 16, True), (3, 208, 16, 0, False), (3, 7, 5, 4, False), (4, 40, 24, 20, True),
                                                  (3, 250, 20, 250, False)])
def test_linear_attention_recalls_a_far_memory(dtype, H, dk, dv, rot, silu):
    """Both forms of the recurrence over 600 tokens in portions, with inputs made so that a fault shows: head 0 keeps
    everything, head 1 nothing but the current token, the others fade; the first token writes along key entry dk - 1, which
    no later key touches and the last token asks for, so head 0's last row is the first token's value and nothing else. A
    second request beside it never writes along that entry. Portions cut at a chunk's edges and just beside them, and
    the tokens whole."""
    from jllm_serve_amd.kernels import ops
    act = act_type(dtype)
    torch.manual_seed(dk)
    T = 600
    decay = [1.0, 0.0] + [0.9, 0.998][:H - 2]
    k_scale = 0.5
    base = 300.0
    last = dk - 1  # beyond the rotated entries, or one side of the slowest pair
    act_in = (lambda t: P.silu(t)) if silu else (lambda t: t)

    def make(writes):
        y = torch.randn(T, 3 + 2 * H * dk + H * dv + 8)
        q, k = y[:, 3:3 + H * dk].view(T, H, dk), y[:, 3 + H * dk:3 + 2 * H * dk].view(T, H, dk)
        if not (rot == dk):
            k[1:, :, last] = 0.0
            k[0] = 0.0
            if writes:
                k[0, :, last] = 3.0
            q[-1] = 0.0
            q[-1, :, last] = 2.0
        return y.to(act)

    reqs = [make(True), make(False)]
    pos = torch.arange(T)

    def plain(y):
        y = y.double()
        q, k = act_in(y[:, 3:3 + H * dk]).view(T, H, dk), act_in(y[:, 3 + H * dk:3 + 2 * H * dk]).view(T, H, dk)
        v = act_in(y[:, 3 + 2 * H * dk:3 + 2 * H * dk + H * dv]).view(T, H, dv)
        if rot:
            q, k = P.rotate_half(q, pos, rot, base), P.rotate_half(k, pos, rot, base)
        return P.decayed_memory(q, k * k_scale, v, decay)[0], v, q, k

    wants = []
    for r, writes in zip(reqs, (True, False)):
        o, v, q, k = plain(r)
        wants.append(o.reshape(T, H * dv))
        if rot != dk:
            far = k_scale * float(q[-1, 0, last] * k[0, 0, last]) * v[0, 0]
            assert torch.allclose(o[-1, 0], far, atol=1e-9), "head 0's last row is the first token's value, or the test is blind"
            assert float(o[-1, 0].abs().max()) > 0.1 if writes else float(o[-1].abs().max()) == 0.0
        assert torch.allclose(o[300, 1], k_scale * (q[300, 1] @ k[300, 1]) * v[300, 1]), "head 1 keeps nothing"
    cos = sin = None
    if rot:
        f = torch.pow(torch.tensor(base, dtype=F64), -2.0 * torch.arange(rot // 2, dtype=F64) / rot)
        ang = pos.double()[:, None] * f[None]
        cos, sin = torch.cos(ang).float().to(DEV), torch.sin(ang).float().to(DEV)
    powers = ops.decay_powers(decay, DEV)

    class Seg:
        def __init__(self, row0, n):
            self.row0, self.n = row0, n
    off = 4 if dk % 16 == 0 else 3  # the rows as a view: an offset that the chunked form takes, and one it does not need to
    for cuts, chunked in (([300, 2, 1, 1, 296], True), ([64, 63, 65, 128, 3, 1, 30, 246], True), ([T], True), ([T], False), ([299, 1, 300], False)):
        state = torch.zeros(5, H, dv, dk, device=DEV)
        slots = torch.tensor([3, 1], dtype=torch.int32, device=DEV)
        got = [[], []]
        at = 0
        ops.reset_stats()
        for n in cuts:
            rows = torch.cat([r[at:at + n] for r in reqs]).to(DEV)
            big = torch.zeros(2 * n, -(-(rows.shape[1] + 4) // 8) * 8, dtype=act, device=DEV)
            big[:, off:off + rows.shape[1] - 3] = rows[:, 3:]
            req, ch = ops.linear_chunk_plan([Seg(0, n), Seg(n, n)])
            plan = dict(requests=torch.tensor(req, dtype=torch.int32, device=DEV), chunks=torch.tensor(ch, dtype=torch.int32, device=DEV)) if chunked else {}
            raw = ops.linear_attention(big, off, off + H * dk, off + 2 * H * dk, powers, state,
                                       torch.tensor([0] * n + [1] * n, dtype=torch.int32, device=DEV), slots, 2, H, dk, dv,
                                       positions=torch.cat([pos[at:at + n]] * 2).to(torch.int32).to(DEV), cos=cos, sin=sin, rot_dims=rot,
                                       silu=silu, k_scale=k_scale, **plan).cpu()
            got[0].append(raw[:n])
            got[1].append(raw[n:])
            at += n
        if chunked and dk % 16 == 0 and dv % 16 == 0 and rot % 8 == 0:
            assert ops.stats()["ran"].get("jllm_linear_chunks", 0) == len(cuts), "the chunked form takes these sizes"
        assert float(state[[0, 2, 4]].abs().max()) == 0.0, "a state row of no request was written"
        for i in range(2):
            out = torch.cat(got[i]).double()
            err = (out - wants[i]).abs().view(T, H, dv).amax(dim=(0, 2))
            size = wants[i].abs().view(T, H, dv).amax(dim=(0, 2))
            assert bool((err <= 2e-5 * size + 1e-6).all()), f"request {i} cuts {cuts} chunked {chunked}: per head {err.tolist()} of {size.tolist()}"
            if rot != dk:  # among sums of hundreds of terms the last row of head 0 is small: held on its own
                assert torch.allclose(out[-1], wants[i][-1], atol=1e-5 * float(wants[i][-1].abs().max()) + 1e-6)


# ------------------------------------------------------------------------------------------------ the attention


def _far_layer(heads, kv, dim, size):
    return {"type": "parallel", "mlp": None, "mixer": {"left": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": 1.5, "mask": {"size": size}},
                                                       "right": {"heads": 1, "dim": 16, "vdim": 16, "decay": [0.9]}}}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads, kv, dim, size", [(4, 2, 32, 37), (3, 3, 20, 37), (8, 2, 64, 128), (6, 1, 48, 130)])
@pytest.mark.parametrize("place", ["first", "last", "page", "middle"])
def test_chunk_attention_finds_one_key_within_its_chunk_and_not_beyond(dtype, heads, kv, dim, size, place, tmp_path):
    """Weights and inputs made so that one key decides: only the row at ``hot`` has a part along input entry 0, and every
    query lies along that row's key. Later rows of its chunk put their weight on it (less with the distance, by the
    head's slope), rows of the next chunk must not see it: at a chunk's first and last position, a page's first, and
    inside; in portions, across chunks, and as single rows."""
    from jllm_serve_amd.engine import build_runner, load_model
    from jllm_serve_amd.engine.step import StepEntry
    from jllm_serve_amd.weights.safetensors_io import write_safetensors
    width, page = 64, 8
    cfg = {"architecture": "Gubotar", "vocab": 50, "width": width, "norm": {"eps": 1e-6}, "layers": [_far_layer(heads, kv, dim, size)]}
    folder = gt.write_model(str(tmp_path / "far"), cfg, 11)
    w = gt.load_weights(folder)
    m = cfg["layers"][0]["mixer"]["left"]
    hot = {"first": size, "last": 2 * size - 1, "page": -(-(size + 1) // page) * page, "middle": size + size // 2}[place]
    g = torch.Generator().manual_seed(5)
    L = "l0.mix.left."
    w[L + "temp"] = torch.linspace(0.8, 1.3, heads, dtype=F64).to(torch.bfloat16).double()
    kw = w[L + "k"]
    kw[:, :2] = 0.0
    kw[:, 0] = (torch.randn(kv * dim, generator=g, dtype=F64)).to(torch.bfloat16).double()
    key = P.rms(kw[:, 0].view(kv, dim) * 8.0, 1e-6) * w[L + "k.norm"]
    qw = w[L + "q"].view(heads, dim, width)
    qw[:, :, 1] = (key / w[L + "q.norm"]).repeat_interleave(heads // kv, dim=0).to(torch.bfloat16).double() * 4.0
    w[L + "q"] = qw.view(heads * dim, width)
    write_safetensors(os.path.join(folder, "model.safetensors"), {k: v.to(torch.bfloat16) for k, v in w.items()})
    w = gt.load_weights(folder)
    T = 3 * size + 5
    act = act_type(dtype)
    h = torch.randn(T, width, generator=g) * 0.3
    h[:, 0] = 0.0
    h[hot, 0] = 8.0
    h[:, 1] = 1.0
    h = h.to(act)
    lw = P.sub(w, L)
    want = P.chunk_attention(h.double(), m, lw, 1e-6)
    h_no = h.clone()
    h_no[hot, 0] = 0.0
    moved = (want - P.chunk_attention(h_no.double(), m, lw, 1e-6)).abs().amax(dim=1)
    end = (hot // size + 1) * size
    assert float(moved[hot:min(end, hot + 40)].min()) > 0.1 * float(want.abs().max()), "the key decides its chunk's later rows, or the test is blind"
    assert float(moved[end:].max()) == 0.0 and float(moved[:hot].max()) == 0.0
    model = load_model(folder, dtype, torch.device(DEV), max_positions=512)
    runner = build_runner(model, page_size=page, pool_tokens=1024, max_requests=2)
    left = model.layers[0].mixer.branches[0]
    w_in = torch.cat([w[L + "q"], w[L + "k"]]).to(act).to(DEV)  # (the shared input product is the parallel mixer's)
    from jllm_serve_amd.kernels import ops
    for cuts in ([T], [size - 1, 2, size - 3, 4, 2] + [1] * 10 + [T - 2 * size - 14], [hot + 1] + [1] * (T - hot - 1)):
        assert sum(cuts) == T
        got, at = [], 0
        for n in cuts:
            ctx = runner.prepare([StepEntry("far", [0] * n, [])])
            y = ops.gemm(h[at:at + n].to(DEV), w_in, out_dtype=act, exact=dtype == "float32")
            slot = model.layers[0].mixer._slot(model.layers[0].states.view(runner.cache.slots[0], 1), 0)
            rows = left.heads_rows_from(y, ctx, slot)
            got.append(ops.gemm(rows, left.output_weight(), out_dtype=torch.float32, exact=dtype == "float32").cpu())
            runner.cache.commit("far", n)
            at += n
        runner.finish("far")
        err = (torch.cat(got).double() - want).abs().amax(dim=1)
        tol = (1e-4 if dtype == "float32" else 3e-2) * float(want.abs().max())
        bad = (err > tol).nonzero().flatten().tolist()
        assert not bad, f"rows at positions {bad[:8]} differ by up to {float(err.max())} (the key is at {hot}, chunks of {size}, cuts {cuts[:6]})"


def test_chunks_and_slopes_in_both_attention_kernels_and_with_shared_key_ranges():
    """The matrix-core kernel against the general one on the same pages, random keys, chunks and contexts in every
    alignment: single rows whose key ranges are shared out over workgroups, and tiles."""
    from jllm_serve_amd.kernels import ops
    torch.manual_seed(9)
    H, G, d, page = 8, 4, 64, 16
    n_pages = 80
    kc = torch.randn(n_pages, G, page, d, device=DEV).to(torch.bfloat16)
    vc = torch.randn(n_pages, G, page, d, device=DEV).to(torch.bfloat16)
    slopes = torch.tensor([2.0 ** (-8 * (h + 1) / H) for h in range(H)], device=DEV)
    for chunk in (1, 50, 64, 96, 200, 1024, 0):
        for cap in (0.0, 3.0):
            lens = [1, 63, 64, 65, 200, 640, 1200]
            table = torch.stack([torch.randperm(n_pages)[:75] for _ in lens]).to(torch.int32).to(DEV).contiguous()
            pos = torch.tensor([n - 1 for n in lens], dtype=torch.int32, device=DEV)
            req = torch.arange(len(lens), dtype=torch.int32, device=DEV)
            q = torch.randn(len(lens), H * d, device=DEV).to(torch.bfloat16)
            tiles = torch.tensor([[r, r, 1, -1] for r in range(len(lens))], dtype=torch.int32, device=DEV).flatten()
            meta = {"tiles_dev": tiles, "n_tiles": len(lens), "single_rows": True, "max_context": 1200}
            args = (q, kc, vc, table, req, pos, H, G, 1, d, d, 0.2)
            kw = dict(softcap=cap, out_dtype=torch.float32, chunk=chunk, slopes=slopes)
            ops.reset_stats()
            a = ops.attention_dv(*args, meta=meta, **kw)
            assert ops.stats()["ran"].get("jllm_attention_dv_bf16") == 1
            b = ops.attention_dv(*args, exact=True, **kw)
            assert float((a - b).abs().max()) < 2e-2, (chunk, cap)
            assert float((b - ops.attention_dv(*args, exact=True, **{**kw, "slopes": None})).abs().max()) > (1e-2 if chunk != 1 else -1)
            # a portion of one request: tiles of up to 128 rows
            T, p0 = 300, 170
            pos = torch.arange(p0, p0 + T, dtype=torch.int32, device=DEV)
            req = torch.zeros(T, dtype=torch.int32, device=DEV)
            q = torch.randn(T, H * d, device=DEV).to(torch.bfloat16)
            tiles = torch.tensor([[0, r, min(128, T - r), p0 + r] for r in range(0, T, 128)], dtype=torch.int32, device=DEV).flatten()
            args = (q, kc, vc, table[:1].contiguous(), req, pos, H, G, 1, d, d, 0.2)
            a = ops.attention_dv(*args, meta={"tiles_dev": tiles, "n_tiles": 3, "single_rows": False, "max_context": p0 + T}, **kw)
            assert ops.stats()["ran"].get("jllm_attention_dv_bf16") == 2
            assert float((a - ops.attention_dv(*args, exact=True, **kw)).abs().max()) < 2e-2, (chunk, cap)


# ------------------------------------------------------------------------------------------------ mixers and models


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_mixers_and_feed_forwards_alone(name, dtype, built, folders):
    """Every layer's mixer on random inputs: a portion from position 0, further portions and single rows from the cache
    and the state; every feed-forward."""
    from jllm_serve_amd.engine.step import StepEntry
    cfg = gt.CONFIGS[name][0]
    eps = cfg["norm"]["eps"]
    w = gt.load_weights(folders[name])
    model, runner = built(name, dtype)
    act = act_type(dtype)
    torch.manual_seed(4)
    cuts = (29, 6, 1, 1, 2, 80, 1, 17)
    T = sum(cuts)
    xs = [(torch.randn(T, cfg["width"]) * 0.8).to(act) for _ in cfg["layers"]]
    pos = torch.arange(T)
    want = [P.mix(x.double(), l, P.sub(w, f"l{i}.mix."), pos, eps) for i, (x, l) in enumerate(zip(xs, cfg["layers"]))]
    got = [[] for _ in xs]
    at = 0
    for n in cuts:
        ctx = runner.prepare([StepEntry("mix", [0] * n, [])])
        for i in range(len(xs)):
            block = model.layers[i]
            got[i].append(block.mixer.output(xs[i][at:at + n].to(DEV), ctx, block.states.view(runner.cache.slots[i], 1)).cpu())
            if block.ffn is not None:
                ff = block.ffn.output(xs[i][at:at + n].to(DEV), ctx)
                close(ff, P.gated_ff(xs[i][at:at + n].double(), P.sub(w, f"l{i}.mlp.")), dtype, f"{name} layer {i} feed-forward, {n} rows")
        runner.cache.commit("mix", n)
        at += n
    runner.finish("mix")
    for i, l in enumerate(cfg["layers"]):
        close(torch.cat(got[i]), want[i], dtype, f"{name} layer {i} {l['type']} mixer")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_stream_after_every_layer(name, dtype, built, folders):
    from jllm_serve_amd.engine.step import StepEntry
    model, runner = built(name, dtype)
    cfg = gt.CONFIGS[name][0]
    toks = gt.prompt(name, 37)
    streams = []
    P.forward(cfg, gt.load_weights(folders[name]), toks, watch=lambda i, x: streams.append(x.clone()))
    cuts = [30, 5, 1, 1]
    got = [[] for _ in streams]
    at = 0
    for n in cuts:
        model.watch = lambda run, x: got[run].append(x.detach().cpu().clone())
        try:
            runner.step([StepEntry("w", toks[at:at + n], [])])
        finally:
            model.watch = None
        at += n
    runner.finish("w")
    for r, s in enumerate(streams):
        tol = (2e-5 if dtype == "float32" else 6e-2) * float(s.abs().max())
        assert float((torch.cat(got[r]).double() - s).abs().max()) <= tol, f"{name} {dtype}: the stream after layer {r}"


def build_trace(name):
    t = replay.Trace(page=gt.CONFIGS[name][2])
    lens = [1, 2, 3, 9, 40, 171]
    toks = {f"r{n}": gt.prompt(name, n) for n in lens}
    longest = toks[f"r{lens[-1]}"]
    replay.whole(t, "whole", longest)
    replay.tail_one_by_one(t, "tail", longest, tail=70)
    replay.portions(t, "cut", longest)
    replay.portions(t, "cut2", longest, sizes=(64, 2, 2, 62, 1, 33))
    for rid, tk in toks.items():
        replay.whole(t, "w" + rid, tk)
    more = dict(toks)
    more["x1"] = gt.prompt(name, 45, seed=1)
    more["x2"] = gt.prompt(name, 2, seed=2)
    more["x3"] = gt.prompt(name, 66, seed=3)
    replay.mixed(t, more, seed=len(name))
    req_tokens = {"whole": longest, "tail": longest, "cut": longest, "cut2": longest, **{"w" + k: v for k, v in toks.items()}, **more}
    return t, req_tokens


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_replay_matches_plain(name, dtype, folders, plain_logits, tmp_path):
    """bin/trace_run: whole, the last tokens one by one, portions down to two tokens, mixed batches with at most four live
    requests on a pool exactly as large as the busiest step (pages and state slots are used again; the free pages are
    reordered before every step)."""
    cfg, _, page = gt.CONFIGS[name]
    trace, req_tokens = build_trace(name)
    got = replay.run(folders[name], dtype, trace, str(tmp_path), page_size=page, max_tokens=trace.peak, shuffle_free=len(name) + 7)
    V = cfg["vocab"]
    ratios = []
    for step, rows in trace.rows.items():
        arr = got[step].reshape(len(rows), V)
        for i, (rid, pos) in enumerate(rows):
            ref = plain_logits(name, req_tokens[rid])[pos]
            err = float(np.abs(arr[i].astype(np.float64) - ref.numpy()).max())
            assert err <= gt.tolerance(dtype, ref), f"{name} {dtype}: step {step} request {rid} position {pos}: {err}"
            ratios.append(err / float(ref.abs().max()))
    assert float(np.median(ratios)) <= gt.typical(dtype), f"{name} {dtype}: median error {np.median(ratios):.3g} of the largest logit"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["GB", "GC"])
def test_long_decoding_and_reused_slots(name, dtype, built, plain_logits):
    """A short prompt, then 230 tokens one by one (bfloat16: through captured steps) beside a second request that joins
    late; then both end and a third request takes over their pages and state rows."""
    from jllm_serve_amd.engine.step import StepEntry
    model, runner = built(name, dtype, graphs=dtype == "bfloat16")
    a, b, c = gt.prompt(name, 240, seed=5), gt.prompt(name, 70, seed=6), gt.prompt(name, 30, seed=7)
    ra, rb, rc = plain_logits(name, a), plain_logits(name, b), plain_logits(name, c)
    close(runner.step([StepEntry("a", a[:10], range(10))]), ra[:10], dtype, "prompt")
    errs = []
    for i in range(10, 240):
        entries = [StepEntry("a", a[i:i + 1], [0])]
        j = i - 90
        if j == 0:
            entries.append(StepEntry("b", b[:20], [19]))
        elif 0 < j and 20 + j - 1 < 70:
            entries.append(StepEntry("b", b[20 + j - 1:20 + j], [0]))
        out = runner.step(entries)
        close(out[0], ra[i], dtype, f"a at {i}")
        errs.append(float((out[0].double().cpu() - ra[i]).abs().max() / ra[i].abs().max()))
        if len(entries) == 2:
            close(out[1], rb[19 if j == 0 else 20 + j - 1], dtype, f"b beside a at {i}")
    assert float(np.median(errs[-30:])) <= gt.typical(dtype), "the error does not grow with the decoded tokens"
    if dtype == "bfloat16":
        assert runner.graphs.replays > 200
    runner.finish("a")
    runner.finish("b")
    close(runner.step([StepEntry("c", c, range(len(c)))]), rc, dtype, "a request on used pages and used state rows")
    runner.finish("c")
    runner.cache.check()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["GA", "GC"])
def test_greedy_generation_through_the_engine(name, dtype, folders):
    """Engine.generate with more requests than places and a pool so small that requests are preempted and computed
    again (their states start from zero again): the tokens of the plain implementation."""
    from jllm_serve_amd.engine import Engine, SchedulerConfig, build_runner, load_model
    from jllm_serve_amd.sampling import SamplingParams
    cfg = gt.CONFIGS[name][0]
    w = gt.load_weights(folders[name])
    model = load_model(folders[name], dtype, torch.device(DEV), max_positions=128)
    runner = build_runner(model, page_size=8, pool_tokens=160, max_requests=3)
    eng = Engine(runner, SchedulerConfig(max_batch_tokens=40, prefill_chunk=16, max_positions=128), eos_token_ids=())
    prompts = [gt.prompt(name, n, seed=9) for n in (1, 5, 23, 40, 12)]
    n_new = 12
    got = [r.tokens for r in eng.generate(prompts, SamplingParams.greedy_params(max_tokens=n_new))]
    for p, g in zip(prompts, got):  # every token is one of the plain implementation's best, given the tokens before it
        assert len(g) == n_new
        ref = P.forward(cfg, w, p + g)
        for i, tok in enumerate(g):
            row = ref[len(p) - 1 + i]
            assert float(row.max() - row[tok]) <= 2 * gt.tolerance(dtype, row), f"token {i} after a prompt of {len(p)}"
    if dtype == "float32":
        want = [P.generate(cfg, w, p, n_new) for p in prompts]
        assert sum(g == x for g, x in zip(got, want)) >= len(prompts) - 1
    runner.cache.check()
    assert not runner.cache.requests


def test_command_line_runs_the_design(folders):
    import subprocess
    import sys
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "jllm"), "run", "--model", folders["GA"], "--dtype", "float32",
                        "--prompt", "3 1 4 1 5", "--max-tokens", "6", "--temp", "0", "--json", "--ctx", "128", "--ignore-eos"],
                       capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    out = json.loads(r.stdout.strip().splitlines()[-1])
    ref = P.forward(gt.G_A, gt.load_weights(folders["GA"]), [3, 1, 4, 1, 5] + out["tokens"])
    assert len(out["tokens"]) == 6
    for i, tok in enumerate(out["tokens"]):
        row = ref[4 + i]
        assert float(row.max() - row[tok]) <= 2 * gt.tolerance("float32", row)
