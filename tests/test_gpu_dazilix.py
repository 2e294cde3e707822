"""Dazilix on the GPU against the plain implementation (tests/plain/dazilix_plain.py): every mechanism alone (the launch
between sublayers that are normed on both sides, q and k prepared with values that are the keys, the router with its bias,
both forms of the recurrence with a decay per key channel on memories that are hundreds of tokens old and on tokens that
forget everything, the attention with one key that decides at chunk and page edges and with scores far below the sink),
mixers through cache and state, whole prompts against token-by-token decoding, portions down to two tokens, mixed batches
on a pool that is used again, the stream after every layer run, long decoding through captured steps, greedy generation
through the engine, and the command line."""
import json
import os

import numpy as np
import pytest
import torch

import dazilix_tiny as dt
import replay
from plain import dazilix_plain as P

pytestmark = pytest.mark.gpu
DEV = "cuda"
F64 = torch.float64
NAMES = sorted(dt.CONFIGS)


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: dt.write_model(str(tmp_path_factory.mktemp("dazilix_" + name)), cfg, seed, middle)
            for name, (cfg, seed, page, middle) in dt.CONFIGS.items()}


@pytest.fixture(scope="module")
def built(folders):
    from jllm_serve_amd.engine import build_runner, load_model
    cache = {}

    def get(name, dtype, graphs=False):
        if (name, dtype, graphs) not in cache:
            model = load_model(folders[name], dtype, torch.device(DEV), max_positions=1024)
            cache[(name, dtype, graphs)] = (model, build_runner(model, page_size=dt.CONFIGS[name][2], pool_tokens=1024,
                                                                max_requests=4, graphs=graphs))
        return cache[(name, dtype, graphs)]
    return get


@pytest.fixture(scope="module")
def plain_logits(folders):
    memo = {}

    def get(name, tokens):
        key = (name, tuple(tokens))
        if key not in memo:
            memo[key] = P.forward(dt.CONFIGS[name][0], dt.load_weights(folders[name]), list(tokens))
        return memo[key]
    return get


def close(got, want, dtype, what=""):
    err = float((got.double().cpu() - want).abs().max())
    assert err <= dt.tolerance(dtype, want), f"{what}: {err} > {dt.tolerance(dtype, want)}"


def act_type(dtype):
    return torch.float32 if dtype == "float32" else torch.bfloat16


# ------------------------------------------------------------------------------------------------ norms, q and k, router


@pytest.mark.parametrize("width", [12, 70, 128, 1000, 1024, 1500, 2048, 3001, 4096, 8192])
def test_launch_between_sublayers(width):
    """x += rms(a) g (or of a weighted sum of two), x += further rows, x += a vector, and the next norm of the new rows,
    each part with and without the others; rows with a stride of their own."""
    from jllm_serve_amd.kernels import ops
    torch.manual_seed(width)
    n, eps, eps2 = 5, 1e-3, 2e-2
    x = torch.randn(n, width) * 2
    a, b = torch.randn(n, width + 8) * 3, torch.randn(n, width + 8) * 0.2
    g, g2, vec = (torch.randn(width) for _ in range(3))
    rows = torch.randn(n, width)
    for branches in (0, 1, 2):
        for more in (False, True):
            for vtype in (None, torch.float32, torch.bfloat16):
                for act in (torch.float32, torch.bfloat16):
                    aa, bb = a.to(act)[:, :width], b.to(act)[:, :width]
                    want = x.double()
                    if branches:
                        t = 0.5 * aa.double() + (0.25 * bb.double() if branches == 2 else 0.0)
                        want = want + P.rms(t, eps) * g.double()
                    if more:
                        want = want + rows.double()
                    if vtype is not None:
                        want = want + vec.to(vtype).double()
                    for out in (None, act):
                        xd = x.to(DEV)
                        kw = dict(a=aa.to(DEV), gain=g.to(DEV), eps=eps, s1=0.5) if branches else {}
                        if branches == 2:
                            kw.update(a2=bb.to(DEV), s2=0.25)
                        got = ops.rms_between(xd, **kw, add_rows=rows.to(DEV) if more else None,
                                              add_vec=vec.to(vtype).to(DEV) if vtype is not None else None,
                                              nxt=(g2.to(DEV), eps2, out) if out is not None else None)
                        what = (branches, more, vtype, act, out)
                        assert torch.allclose(xd.cpu().double(), want, atol=3e-5, rtol=1e-5), what
                        if out is None:
                            assert got is None
                            continue
                        normed = P.rms(want, eps2) * g2.double()
                        exact = out == torch.float32
                        assert got.dtype == out and torch.allclose(got.cpu().double(), normed, atol=3e-5 if exact else 2e-2, rtol=1e-5 if exact else 1e-2), what


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H, G, dk, dims", [(6, 2, 14, 6), (3, 3, 10, 10), (16, 8, 128, 64), (4, 1, 64, 64), (8, 2, 32, 0), (5, 5, 48, 16), (40, 8, 128, 128), (2, 1, 24, 12)])
@pytest.mark.parametrize("tied", [True, False])
def test_q_and_k_normed_over_the_whole_projection(dtype, H, G, dk, dims, tied):
    """Norm over all of q and all of k, rotation of a head's halves (and of neighbours), values that are the raw keys or
    columns of their own, stores into shuffled pages: rows of every size, whichever kernel takes them."""
    from jllm_serve_amd.kernels import ops
    torch.manual_seed(dk + H)
    act = act_type(dtype)
    page, T, dv = 4, 23, dk if tied else dk + 8
    nq, nk = H * dk, G * dk
    cols = nq + nk + (0 if tied else G * dv)
    y = (torch.randn(T, -(-cols // 16) * 16) * torch.linspace(0.3, 2.0, T)[:, None]).to(act)
    gq, gk = torch.randn(nq) * 0.2 + 1, torch.randn(nk) * 0.2 + 1
    positions = torch.arange(5, 5 + T)
    slots = torch.randperm(8 * page)[:T].int()
    slots[4] = -1
    half = dims // 2
    ang = torch.arange(64, dtype=F64)[:, None] * torch.pow(torch.tensor(50.0, dtype=F64), -2.0 * torch.arange(max(half, 1), dtype=F64) / max(dims, 1))[None]
    cos, sin = torch.cos(ang).float().to(DEV), torch.sin(ang).float().to(DEV)
    tol = dict(atol=2e-5, rtol=1e-5) if dtype == "float32" else dict(atol=2e-2, rtol=1e-2)
    for pairing in ("half", "interleaved"):
        yd = y.clone().to(DEV)
        kc = torch.zeros(8, G, page, dk, device=DEV, dtype=act)
        vc = torch.zeros(8, G, page, dv, device=DEV, dtype=act)
        ops.qkv_prepare(yd, positions.int().to(DEV), slots.to(DEV), H, G, 1, dk, dv, kc, vc, gq=gq.to(DEV), gk=gk.to(DEV), eps=1e-3,
                        cos=cos if dims else None, sin=sin if dims else None, rot_dims=dims, pairing=pairing, tied_values=tied)
        q = (P.rms(y[:, :nq].double(), 1e-3) * gq.double()).view(T, H, dk)
        k = (P.rms(y[:, nq:nq + nk].double(), 1e-3) * gk.double()).view(T, G, dk)
        if dims and pairing == "half":
            q, k = P.rotate_half(q, positions, dims, 50.0), P.rotate_half(k, positions, dims, 50.0)
        elif dims:  # neighbours: the same with the entries' order changed
            order = torch.cat([torch.arange(0, dims, 2), torch.arange(1, dims, 2), torch.arange(dims, dk)])
            back = torch.argsort(order)
            q = P.rotate_half(q[..., order], positions, dims, 50.0)[..., back]
            k = P.rotate_half(k[..., order], positions, dims, 50.0)[..., back]
        assert torch.allclose(yd[:, :nq].cpu().double(), q.reshape(T, nq), **tol), pairing
        assert torch.equal(yd[:, nq:].cpu(), y[:, nq:])
        raw = (y[:, nq:nq + nk] if tied else y[:, nq + nk:nq + nk + G * dv]).reshape(T, G, dv)
        for t in range(T):
            s = int(slots[t])
            if s < 0:
                continue
            assert torch.allclose(kc[s // page, :, s % page].cpu().double(), k[t], **tol), (pairing, t)
            assert torch.equal(vc[s // page, :, s % page].cpu(), raw[t]), (pairing, t)
        assert int((kc != 0).any(dim=-1).sum()) == (T - 1) * G and int((vc != 0).any(dim=-1).sum()) == (T - 1) * G


@pytest.mark.parametrize("E, top", [(1, 1), (2, 1), (5, 5), (12, 3), (64, 8), (65, 9), (128, 2), (200, 70), (256, 256), (300, 4)])
def test_router_softmaxes_the_chosen_logits(E, top):
    """Choice by the largest logits, weights from the softmax over those alone (up to 256 experts in registers, beyond
    that the general kernel); also sigmoid scores with a correction."""
    from jllm_serve_amd.kernels import ops
    g = torch.Generator().manual_seed(E * 100 + top)
    T = 257
    z = torch.randn(T, E, generator=g) * 3.0
    want_e, want_w = P.choose(z.double(), top)
    got_e, got_w = ops.moe_router(z.to(DEV), None, 1, 1, top, 1.0, score="softmax", normalize=True)
    got_e, got_w = got_e.cpu().long(), got_w.cpu().double()
    same = (got_e == want_e).all(dim=1)
    if top < 32:
        assert int((~same).sum()) <= 1, "fp32 and float64 may order one near-tie differently"
    dense = lambda e, w: torch.zeros(T, E, dtype=F64).scatter_(1, e, w)
    assert float((dense(got_e, got_w) - dense(want_e, want_w))[same].abs().max()) < 1e-6
    assert torch.allclose(got_w.sum(dim=1), torch.ones(T, dtype=F64), atol=1e-5) and all(len(set(r.tolist())) == top for r in got_e)
    corr = torch.randn(E, generator=g)
    s = torch.sigmoid(z.double())
    want_e = torch.topk(s + corr.double(), top, dim=1).indices
    got_e, got_w = ops.moe_router(z.to(DEV), corr.to(DEV), 1, 1, top, 2.5)
    w = torch.gather(s, 1, got_e.cpu().long())
    assert torch.allclose(got_w.cpu().double(), 2.5 * w / (w.sum(dim=1, keepdim=True) + 1e-20), atol=1e-5)
    if top < 32:
        assert int((got_e.cpu().long() != want_e).any(dim=1).sum()) <= 2


# ------------------------------------------------------------------------------------------------ the recurrence


class Seg:
    def __init__(self, row0, n):
        self.row0, self.n = row0, n


def _run_recurrence(reqs, cuts, chunked, act, H, dk, dv, w_up, bias, rank, k_scale, tau, off, state=None):
    """The requests' rows [T, q | k | v | middle] through the kernels in portions; returns (outputs per request, state)."""
    from jllm_serve_amd.kernels import ops
    n_req = len(reqs)
    if state is None:
        state = torch.zeros(2 * n_req + 1, H, dv, dk, device=DEV)
    slots = torch.tensor([2 * i + 1 for i in range(n_req)][::-1], dtype=torch.int32, device=DEV)
    got = [[] for _ in reqs]
    at = 0
    width = reqs[0].shape[1]
    m_off = off + 2 * H * dk + H * dv
    for n in cuts:
        rows = torch.cat([r[at:at + n] for r in reqs]).to(DEV)
        big = torch.zeros(n_req * n, -(-(width + off) // 16) * 16, dtype=act, device=DEV)
        big[:, off:off + width] = rows
        req, ch = ops.linear_chunk_plan([Seg(i * n, n) for i in range(n_req)])
        plan = dict(requests=torch.tensor(req, dtype=torch.int32, device=DEV), chunks=torch.tensor(ch, dtype=torch.int32, device=DEV)) if chunked else {}
        raw = ops.linear_attention(big, off, off + H * dk, off + 2 * H * dk, None, state,
                                   torch.tensor([i for i in range(n_req) for _ in range(n)], dtype=torch.int32, device=DEV), slots, n_req, H, dk, dv,
                                   k_scale=k_scale, decay_off=m_off, decay_up=w_up, decay_bias=bias, decay_rank=rank, tau=tau, **plan).cpu()
        for i in range(n_req):
            got[i].append(raw[i * n:(i + 1) * n])
        at += n
    assert float(state[0::2].abs().max()) == 0.0, "a state row of no request was written"
    return [torch.cat(g).double() for g in got], state


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H, dk, dv, rank, tau", [(3, 16, 16, 1, 1.0), (3, 64, 48, 16, 3.0), (4, 128, 128, 16, 16.0), (3, 256, 256, 40, 8.0), (3, 48, 176, 7, 0.5),
                                                  (3, 208, 16, 64, 2.0), (3, 7, 5, 3, 1.0), (4, 40, 24, 16, 5.0), (3, 250, 20, 33, 4.0)])
def test_channel_decay_recalls_a_far_memory(dtype, H, dk, dv, rank, tau):
    """Both forms of the recurrence over 600 tokens in portions, with inputs made so that a fault shows. Head 0's last key
    channel fades by a number per token that its bias gives (a factor of about e over the whole sequence), head 1 forgets
    everything with every token, in the other channels the tokens choose. The first token writes along channel dk - 1, which
    no later key touches and the last token asks for: head 0's last row is the first token's value times the product of all
    599 later decays and nothing else. A second request beside it never writes along that channel. Portions cut at a chunk's
    edges and just beside them, and the tokens whole."""
    from jllm_serve_amd.kernels import ops
    act = act_type(dtype)
    torch.manual_seed(dk)
    T, k_scale, last = 600, 0.5, dk - 1
    full = -(-rank // ops.LINEAR_MIDDLE) * ops.LINEAR_MIDDLE
    w_up = torch.zeros(H * dk, full)
    w_up[:, :rank] = torch.randn(H * dk, rank) * 2.0 * rank ** -0.5
    bias = torch.randn(H * dk) * 2.0 + 1.0
    fade = float(np.log(1.0 / np.expm1(tau / T)))  # softplus(-fade) = tau / T: sigmoid(fade)^(1 / tau) = exp(-1 / T)
    for h in range(H):
        w_up[h * dk + last] = 0.0
        bias[h * dk + last] = fade
    w_up[dk:2 * dk] = 0.0
    bias[dk:2 * dk] = -150.0 * max(tau, 1.0)
    w_up = w_up.to(act)

    def make(writes):
        y = torch.randn(T, 2 * H * dk + H * dv + full)
        y[:, 2 * H * dk + H * dv + rank:] = 0.0
        q, k = y[:, :H * dk].view(T, H, dk), y[:, H * dk:2 * H * dk].view(T, H, dk)
        k[1:, :, last] = 0.0
        k[0] = 0.0
        if writes:
            k[0, :, last] = 3.0
        q[-1] = 0.0
        q[-1, :, last] = 2.0
        return y.to(act)

    reqs = [make(True), make(False)]

    def plain(y):
        y = y.double()
        q, k = y[:, :H * dk].view(T, H, dk), y[:, H * dk:2 * H * dk].view(T, H, dk) * k_scale
        v = y[:, 2 * H * dk:2 * H * dk + H * dv].view(T, H, dv)
        z = y[:, 2 * H * dk + H * dv:] @ w_up.double().t() + bias.double()
        return P.channel_memory(q, k, v, P.channel_decay(z, tau).view(T, H, dk))[0], v

    wants = []
    for r, writes in zip(reqs, (True, False)):
        o, v = plain(r)
        wants.append(o.reshape(T, H * dv))
        far = k_scale * 6.0 * np.exp(-(T - 1) / T) * v[0, 0] * (1.0 if writes else 0.0)
        assert torch.allclose(o[-1, 0], far, atol=1e-6), "head 0's last row is the faded first token's value, or the test is blind"
        assert float(o[-1, 1].abs().max()) < 1e-9, "head 1 keeps nothing"
    for cuts, chunked in (([300, 2, 1, 1, 296], True), ([64, 63, 65, 128, 3, 1, 30, 246], True), ([T], True), ([T], False), ([299, 1, 300], False)):
        off = 8 if chunked else 3  # the rows as a view: an offset that the chunked form takes, and one it does not need to
        ops.reset_stats()
        got, _ = _run_recurrence(reqs, cuts, chunked, act, H, dk, dv, w_up.to(DEV), bias.to(DEV), rank, k_scale, tau, off)
        if chunked and dk % 16 == 0 and dv % 16 == 0:
            assert ops.stats()["ran"].get("jllm_linear_chunks", 0) == len(cuts), "the chunked form takes these sizes"
        for i in range(2):
            err = (got[i] - wants[i]).abs().view(T, H, dv).amax(dim=(0, 2))
            size = wants[i].abs().view(T, H, dv).amax(dim=(0, 2))
            assert bool((err <= 3e-5 * size + 1e-6).all()), f"request {i} cuts {cuts} chunked {chunked}: per head {err.tolist()} of {size.tolist()}"
            # among sums of hundreds of terms the last row of head 0 is small: held on its own
            assert torch.allclose(got[i][-1], wants[i][-1], atol=3e-5 * float(wants[i][-1].abs().max()) + 1e-6), (cuts, chunked)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H, dk, dv", [(2, 16, 16), (2, 64, 64), (1, 128, 48), (1, 192, 32)])
def test_tokens_that_forget_everything(dtype, H, dk, dv):
    """Decays down to exactly 0 and up to exactly 1 at single tokens, at every place within a chunk and a tile, among
    ordinary ones: nothing overflows, what lies before such a token is gone and what comes after it is exact. Both forms
    agree with the plain recurrence to fp32 rounding, row by row."""
    act = act_type(dtype)
    torch.manual_seed(dk + 1)
    T, rank, full, tau = 300, 2, 32, 1.0
    y = torch.randn(T, 2 * H * dk + H * dv + full)
    m = y[:, 2 * H * dk + H * dv:]
    m[:] = 0.0
    m[:, 0] = torch.randn(T)
    hit = torch.zeros(T, dtype=torch.bool)
    hit[torch.tensor([0, 1, 15, 16, 17, 31, 47, 63, 64, 65, 66, 100, 127, 128, 129, 190, 191, 240, 299])] = True
    m[hit, 1] = 1.0
    y = y.to(act)
    w_up = torch.zeros(H * dk, full)
    w_up[:, 0] = torch.randn(H * dk)
    # where the token hits: the even channels forget everything (z near -600), the odd ones keep everything (z near 600)
    w_up[:, 1] = torch.where(torch.arange(H * dk) % 2 == 0, -600.0, 600.0)
    w_up = w_up.to(act)
    bias = torch.full((H * dk,), 1.5)
    d = y.double()
    q, k = d[:, :H * dk].view(T, H, dk), d[:, H * dk:2 * H * dk].view(T, H, dk)
    v = d[:, 2 * H * dk:2 * H * dk + H * dv].view(T, H, dv)
    alpha = P.channel_decay(d[:, 2 * H * dk + H * dv:] @ w_up.double().t() + bias.double(), tau)
    assert float(alpha[15, 0]) < 1e-200 and float(alpha[15, 1]) == 1.0
    want = P.channel_memory(q, k, v, alpha.view(T, H, dk))[0].reshape(T, H * dv)
    for cuts, chunked in (([T], True), ([65, 66, 169], True), ([T], False), ([1] * 20 + [280], True)):
        got, _ = _run_recurrence([y], cuts, chunked, act, H, dk, dv, w_up.to(DEV), bias.to(DEV), rank, 1.0, tau, 8)
        assert bool(torch.isfinite(got[0]).all()), (cuts, chunked)
        err, size = (got[0] - want).abs().amax(dim=1), want.abs().amax(dim=1)
        bad = (err > 3e-5 * size.max() + 1e-6).nonzero().flatten().tolist()
        assert not bad, f"cuts {cuts[:3]} chunked {chunked}: rows {bad[:8]}, {float(err.max())} of {float(size.max())}"


# ------------------------------------------------------------------------------------------------ the attention


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads, kv, dim, size", [(4, 2, 32, 37), (3, 3, 20, 37), (8, 2, 64, 128), (6, 1, 48, 130)])
@pytest.mark.parametrize("place", ["first", "last", "page", "middle"])
def test_attention_finds_one_key_within_its_chunk_and_not_beyond(dtype, heads, kv, dim, size, place, tmp_path):
    """Weights and inputs made so that one key decides: only the row at ``hot`` has a part along input entry 0, and every
    query lies along that row's key, in the entries that rotation leaves alone. Later rows of its chunk put their weight on
    it, rows of the next chunk must not see it: at a chunk's first and last position, a page's first, and inside; in
    portions, across chunks, and as single rows."""
    from jllm_serve_amd.engine import build_runner, load_model
    from jllm_serve_amd.engine.step import StepEntry
    from jllm_serve_amd.weights.safetensors_io import write_safetensors
    width, page, dims = 64, 8, 4
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": 0.6, "mask": {"size": size}, "rot": {"base": 100.0, "dims": dims}}
    cfg = {"architecture": "Dazilix", "vocab": 50, "width": width, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
           "layers": [{"type": "attention", "mixer": m, "mlp": None}]}
    folder = dt.write_model(str(tmp_path / "far"), cfg, 11)
    w = dt.load_weights(folder)
    hot = {"first": size, "last": 2 * size - 1, "page": -(-(size + 1) // page) * page, "middle": size + size // 2}[place]
    g = torch.Generator().manual_seed(5)
    L = "l0.mix."
    kw = w[L + "k"]
    kw[:, :2] = 0.0
    along = torch.randn(kv, dim, generator=g, dtype=F64)
    along[:, :dims] = 0.0
    kw[:, 0] = along.view(-1).to(torch.bfloat16).double()
    key = P.rms(kw[:, 0] * 8.0, 1e-6) * w[L + "k.norm"]
    qw = w[L + "q"].view(heads, dim, width)
    qw[:, :, 1] = (key.view(kv, dim).repeat_interleave(heads // kv, dim=0) / w[L + "q.norm"].view(heads, dim)).to(torch.bfloat16).double() * 4.0
    w[L + "q"] = qw.view(heads * dim, width)
    write_safetensors(os.path.join(folder, "model.safetensors"), {k: v.to(torch.bfloat16) for k, v in w.items()})
    w = dt.load_weights(folder)
    T = 3 * size + 5
    act = act_type(dtype)
    h = torch.randn(T, width, generator=g) * 0.3
    h[:, 0] = 0.0
    h[hot, 0] = 8.0
    h[:, 1] = 1.0
    h = h.to(act)
    lw, pos = P.sub(w, L), torch.arange(T)
    want = P.chunk_attention(h.double(), m, lw, pos, 1e-6)
    h_no = h.clone()
    h_no[hot, 0] = 0.0
    moved = (want - P.chunk_attention(h_no.double(), m, lw, pos, 1e-6)).abs().amax(dim=1)
    end = (hot // size + 1) * size
    assert float(moved[hot:end].min()) > 0.1 * float(want.abs().max()), "the key decides its chunk's later rows, or the test is blind"
    assert float(moved[end:].max()) == 0.0 and float(moved[:hot].max()) == 0.0
    model = load_model(folder, dtype, torch.device(DEV), max_positions=512)
    runner = build_runner(model, page_size=page, pool_tokens=1024, max_requests=2)
    mixer = model.layers[0].mixer
    for cuts in ([T], [size - 1, 2, size - 3, 4, 2] + [1] * 10 + [T - 2 * size - 14], [hot + 1] + [1] * (T - hot - 1)):
        assert sum(cuts) == T
        got, at = [], 0
        for n in cuts:
            ctx = runner.prepare([StepEntry("far", [0] * n, [])])
            got.append(mixer.output(h[at:at + n].to(DEV), ctx, runner.cache.slots[0]).cpu())
            runner.cache.commit("far", n)
            at += n
        runner.finish("far")
        err = (torch.cat(got).double() - want).abs().amax(dim=1)
        tol = (1e-4 if dtype == "float32" else 3e-2) * float(want.abs().max())
        bad = (err > tol).nonzero().flatten().tolist()
        assert not bad, f"rows at positions {bad[:8]} differ by up to {float(err.max())} (the key is at {hot}, chunks of {size}, cuts {cuts[:6]})"


def test_a_one_in_the_denominator_with_scores_of_every_size():
    """Both attention kernels with a plain sink on the same pages: scores around 0, far above and far below the sink's,
    single rows whose key ranges are shared out over workgroups and merged, and tiles; against the plain softmax."""
    from jllm_serve_amd.kernels import ops
    torch.manual_seed(9)
    H, G, d, page = 8, 4, 64, 16
    n_pages = 80
    kc = torch.randn(n_pages, G, page, d, device=DEV).to(torch.bfloat16)
    vc = torch.randn(n_pages, G, page, d, device=DEV).to(torch.bfloat16)
    sinks = torch.zeros(H, device=DEV)
    lens = [1, 63, 64, 65, 200, 640, 1200]
    table = torch.stack([torch.randperm(n_pages)[:75] for _ in lens]).to(torch.int32).to(DEV).contiguous()
    for chunk in (1, 50, 96, 1024):
        for shift in (0.0, 40.0, -40.0, -3000.0):
            # every query's first entry meets the keys' first entry, which is 1: all scores move by `shift`
            kc[..., 0] = 1.0
            pos = torch.tensor([n - 1 for n in lens], dtype=torch.int32, device=DEV)
            req = torch.arange(len(lens), dtype=torch.int32, device=DEV)
            q = torch.randn(len(lens), H, d, device=DEV).to(torch.bfloat16)
            q[..., 0] = shift / 0.125
            tiles = torch.tensor([[r, r, 1, -1] for r in range(len(lens))], dtype=torch.int32, device=DEV).flatten()
            meta = {"tiles_dev": tiles, "n_tiles": len(lens), "single_rows": True, "max_context": 1200}
            args = (q.view(len(lens), H * d), kc, vc, table, req, pos, H, G, 1, d, d, 0.125)
            kw = dict(out_dtype=torch.float32, chunk=chunk, sinks=sinks)
            ops.reset_stats()
            a = ops.attention_dv(*args, meta=meta, **kw).cpu().double()
            assert ops.stats()["ran"].get("jllm_attention_dv_bf16") == 1
            fin = ops.heads_finish(ops.attention_dv(*args, meta=meta, defer_merge=True, **kw), H, 1, d, torch.float32).cpu().double()
            b = ops.attention_dv(*args, exact=True, **kw).cpu().double()
            for r, n in enumerate(lens):
                lo = (n - 1) // chunk * chunk
                idx = torch.arange(lo, n)
                pages = table[r].cpu().long()[idx // page]
                K = kc.cpu()[pages, :, idx % page].double()
                V = vc.cpu()[pages, :, idx % page].double()
                for h in range(H):
                    s = (K[:, h // 2] @ q[r, h].cpu().double() * 0.125)[None]
                    want = P.softmax_plus_one(s, torch.ones_like(s, dtype=torch.bool))[0] @ V[:, h // 2]
                    for got, what, tol in ((a, "matrix cores", 2e-2), (fin, "merged while finishing", 2e-2), (b, "general", 1e-5)):
                        err = float((got[r, h * d:(h + 1) * d] - want).abs().max())
                        assert err < tol * max(1.0, float(want.abs().max())), (what, chunk, shift, n, h, err)
                    if shift == -3000.0:
                        assert float(want.abs().max()) == 0.0


# ------------------------------------------------------------------------------------------------ mixers and models


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_mixers_and_feed_forwards_alone(name, dtype, built, folders):
    """Every layer's mixer on random inputs: a portion from position 0, further portions and single rows from the cache
    and the state; every feed-forward (in bfloat16 rows whose router's choice is a close call are left out)."""
    from jllm_serve_amd.engine.step import StepEntry
    cfg = dt.CONFIGS[name][0]
    eps = cfg["norm"]["eps"]
    w = dt.load_weights(folders[name])
    model, runner = built(name, dtype)
    act = act_type(dtype)
    torch.manual_seed(4)
    cuts = (29, 6, 1, 1, 2, 80, 1, 17)
    T = sum(cuts)
    xs = [(torch.randn(T, cfg["width"]) * 0.8).to(act) for _ in cfg["layers"]]
    pos = torch.arange(T)
    want = [P.mix(x.double(), l, P.sub(w, f"l{i}.mix."), pos, eps) for i, (x, l) in enumerate(zip(xs, cfg["layers"]))]
    first_run = {i: r for r, (i, _) in reversed(list(enumerate(P.runs(cfg))))}
    got = [[] for _ in xs]
    at = 0
    for n in cuts:
        ctx = runner.prepare([StepEntry("mix", [0] * n, [])])
        for i, l in enumerate(cfg["layers"]):
            block = model.layers[i]
            x = xs[i][at:at + n]
            got[i].append(block.mixer.output(x.to(DEV), ctx, runner.cache.slots[first_run[i]]).cpu())
            if block.ffn is not None:
                lw = P.sub(w, f"l{i}.mlp.")
                top = l["mlp"]["router"]["top"]
                z = torch.sort(P.linear(x.double(), lw["router"]) + lw["router.b"], dim=1, descending=True).values
                clear = torch.ones(n, dtype=torch.bool) if top == z.shape[1] else (z[:, top - 1] - z[:, top]) > 1e-4
                ff = block.ffn.output(x.to(DEV), ctx).cpu()
                close(ff[clear], P.experts(x.double(), l["mlp"], lw)[clear], dtype, f"{name} layer {i} feed-forward, {n} rows")
        runner.cache.commit("mix", n)
        at += n
    runner.finish("mix")
    for i, l in enumerate(cfg["layers"]):
        close(torch.cat(got[i]), want[i], dtype, f"{name} layer {i} {l['type']} mixer")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_stream_after_every_run(name, dtype, built, folders):
    """The stream behind every run, and the same logits with and without a watcher (which takes the launches between two
    passes apart)."""
    from jllm_serve_amd.engine.step import StepEntry
    model, runner = built(name, dtype)
    cfg = dt.CONFIGS[name][0]
    toks = dt.prompt(name, 37)
    streams = []
    P.forward(cfg, dt.load_weights(folders[name]), toks, watch=lambda i, x: streams.append(x.clone()))
    cuts = [30, 5, 1, 1]
    got = [[] for _ in streams]
    logits = {}
    for watched in (True, False):
        at = 0
        for n in cuts:
            model.watch = (lambda run, x: got[run].append(x.detach().cpu().clone())) if watched else None
            try:
                logits.setdefault(watched, []).append(runner.step([StepEntry("w", toks[at:at + n], range(n))]).cpu())
            finally:
                model.watch = None
            at += n
        runner.finish("w")
    for r, s in enumerate(streams):
        err = (torch.cat(got[r]).double() - s).abs().amax(dim=1)
        tol = (3e-5 if dtype == "float32" else 8e-2) * float(s.abs().max())
        assert float(err.median()) <= tol / 4 and float(err.max()) <= (tol if dtype == "float32" else 2 * tol), f"{name} {dtype}: the stream after run {r}: {float(err.max())}"
    a, b = torch.cat(logits[True]), torch.cat(logits[False])
    assert float((a - b).abs().max()) <= (1e-5 if dtype == "float32" else 3e-2) * float(a.abs().max())


def build_trace(name):
    t = replay.Trace(page=dt.CONFIGS[name][2])
    lens = [1, 2, 3, 9, 40, 171]
    toks = {f"r{n}": dt.prompt(name, n) for n in lens}
    longest = toks[f"r{lens[-1]}"]
    replay.whole(t, "whole", longest)
    replay.tail_one_by_one(t, "tail", longest, tail=70)
    replay.portions(t, "cut", longest)
    replay.portions(t, "cut2", longest, sizes=(64, 2, 2, 62, 1, 33))
    for rid, tk in toks.items():
        replay.whole(t, "w" + rid, tk)
    more = dict(toks)
    more["x1"] = dt.prompt(name, 45, seed=1)
    more["x2"] = dt.prompt(name, 2, seed=2)
    more["x3"] = dt.prompt(name, 66, seed=3)
    replay.mixed(t, more, seed=len(name))
    req_tokens = {"whole": longest, "tail": longest, "cut": longest, "cut2": longest, **{"w" + k: v for k, v in toks.items()}, **more}
    return t, req_tokens


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_replay_matches_plain(name, dtype, folders, plain_logits, tmp_path):
    """bin/trace_run: whole, the last tokens one by one, portions down to two tokens, mixed batches with at most four live
    requests on a pool exactly as large as the busiest step (pages and state slots are used again; the free pages are
    reordered before every step)."""
    cfg, _, page, _ = dt.CONFIGS[name]
    trace, req_tokens = build_trace(name)
    got = replay.run(folders[name], dtype, trace, str(tmp_path), page_size=page, max_tokens=trace.peak, shuffle_free=len(name) + 7)
    V = cfg["vocab"]
    ratios, over = [], []
    for step, rows in trace.rows.items():
        arr = got[step].reshape(len(rows), V)
        for i, (rid, pos) in enumerate(rows):
            ref = plain_logits(name, req_tokens[rid])[pos]
            err = float(np.abs(arr[i].astype(np.float64) - ref.numpy()).max())
            if err > dt.tolerance(dtype, ref):
                over.append((step, rid, pos, err))
            ratios.append(err / float(ref.abs().max()))
    assert len(over) <= dt.turned(dtype, len(ratios)), f"{name} {dtype}: {len(over)} of {len(ratios)} rows, first (step, request, position, error) {over[:3]}"
    assert float(np.median(ratios)) <= dt.typical(dtype), f"{name} {dtype}: median error {np.median(ratios):.3g} of the largest logit"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["DB", "DC"])
def test_long_decoding_and_reused_slots(name, dtype, built, plain_logits):
    """A short prompt, then 230 tokens one by one (bfloat16: through captured steps) beside a second request that joins
    late; then both end and a third request takes over their pages and state rows."""
    from jllm_serve_amd.engine.step import StepEntry
    model, runner = built(name, dtype, graphs=dtype == "bfloat16")
    a, b, c = dt.prompt(name, 240, seed=5), dt.prompt(name, 70, seed=6), dt.prompt(name, 30, seed=7)
    ra, rb, rc = plain_logits(name, a), plain_logits(name, b), plain_logits(name, c)
    ratio = lambda got, ref: float((got.double().cpu() - ref).abs().max() / ref.abs().max())
    errs = {"a": [ratio(x, r) for x, r in zip(runner.step([StepEntry("a", a[:10], range(10))]), ra[:10])], "b": []}
    for i in range(10, 240):
        entries = [StepEntry("a", a[i:i + 1], [0])]
        j = i - 90
        if j == 0:
            entries.append(StepEntry("b", b[:20], [19]))
        elif 0 < j and 20 + j - 1 < 70:
            entries.append(StepEntry("b", b[20 + j - 1:20 + j], [0]))
        out = runner.step(entries)
        errs["a"].append(ratio(out[0], ra[i]))
        if len(entries) == 2:
            errs["b"].append(ratio(out[1], rb[19 if j == 0 else 20 + j - 1]))
    if dtype == "bfloat16":
        assert runner.graphs.replays > 200
    runner.finish("a")
    runner.finish("b")
    errs["c"] = [ratio(x, r) for x, r in zip(runner.step([StepEntry("c", c, range(len(c)))]), rc)]
    runner.finish("c")
    bound = 1e-4 if dtype == "float32" else 0.1
    for who, e in errs.items():
        over = [i for i, v in enumerate(e) if v > bound]
        assert len(over) <= dt.turned(dtype, len(e)), f"{who}: rows {over[:5]}, {max(e)}"
        assert float(np.median(e)) <= dt.typical(dtype), who
    assert float(np.median(errs["a"][-30:])) <= dt.typical(dtype), "the error does not grow with the decoded tokens"
    runner.cache.check()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["DA", "DC"])
def test_greedy_generation_through_the_engine(name, dtype, folders):
    """Engine.generate with more requests than places and a pool so small that requests are preempted and computed
    again (their states start from zero again): the tokens of the plain implementation."""
    from jllm_serve_amd.engine import Engine, SchedulerConfig, build_runner, load_model
    from jllm_serve_amd.sampling import SamplingParams
    cfg = dt.CONFIGS[name][0]
    w = dt.load_weights(folders[name])
    model = load_model(folders[name], dtype, torch.device(DEV), max_positions=128)
    runner = build_runner(model, page_size=8, pool_tokens=160, max_requests=3)
    eng = Engine(runner, SchedulerConfig(max_batch_tokens=40, prefill_chunk=16, max_positions=128), eos_token_ids=())
    prompts = [dt.prompt(name, n, seed=9) for n in (1, 5, 23, 40, 12)]
    n_new = 12
    got = [r.tokens for r in eng.generate(prompts, SamplingParams.greedy_params(max_tokens=n_new))]
    worse = 0
    for p, g in zip(prompts, got):  # every token is one of the plain implementation's best, given the tokens before it
        assert len(g) == n_new
        ref = P.forward(cfg, w, p + g)
        for i, tok in enumerate(g):
            row = ref[len(p) - 1 + i]
            worse += float(row.max() - row[tok]) > 2 * dt.tolerance(dtype, row)
    assert worse <= (0 if dtype == "float32" else 1), f"{worse} tokens that are not among the plain implementation's best"
    if dtype == "float32":
        want = [P.generate(cfg, w, p, n_new) for p in prompts]
        assert sum(g == x for g, x in zip(got, want)) >= len(prompts) - 1
    runner.cache.check()
    assert not runner.cache.requests


def test_command_line_runs_the_design(folders):
    import subprocess
    import sys
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "jllm"), "run", "--model", folders["DA"], "--dtype", "float32",
                        "--prompt", "3 1 4 1 5", "--max-tokens", "6", "--temp", "0", "--json", "--ctx", "128", "--ignore-eos"],
                       capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    out = json.loads(r.stdout.strip().splitlines()[-1])
    ref = P.forward(dt.D_A, dt.load_weights(folders["DA"]), [3, 1, 4, 1, 5] + out["tokens"])
    assert len(out["tokens"]) == 6
    for i, tok in enumerate(out["tokens"]):
        row = ref[4 + i]
        assert float(row.max() - row[tok]) <= 2 * dt.tolerance("float32", row)
