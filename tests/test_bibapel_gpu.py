"""Bibapel on the GPU kernels against the plain implementation (bibapel_oracle): each mechanism alone, then whole models
through the engine's feeds, scheduler and graphs."""
import math

import pytest
import torch

import bibapel_models as S
import bibapel_oracle as O
from stack_helpers import DT, act, engine, relerr, rnd, run_rows, st

pytestmark = pytest.mark.gpu
# Whole models: row errors (sekolorn_models.error), largest and for 19 rows of 20. Unit norms and per-head norms magnify the
# rounding of a row whose values nearly cancel ahead of them, hence the two bounds in bf16.
WHOLE = {"f32": (2e-5, 1e-5), "bf16": (0.1, 0.04)}
TOL = {"f32": 3e-5, "bf16": 1.5e-2}


@pytest.fixture(scope="module")
def K(gpu):
    from nats_llm_studio_amd.ops import stack
    stack.lib()
    return stack


def load(tmp_path, cfg, W, dt, ctx=1024):
    from nats_llm_studio_amd.models.registry import load_model
    return load_model(S.write_model(str(tmp_path / "model"), cfg, W), "cuda:0", dtype=DT[dt], ctx=ctx)


def close(got, want, dt):
    e = S.error(got, want), S.error(got, want, 0.95)
    print(f"{len(got)} rows: error {e[0]:.3g}, 19 of 20 {e[1]:.3g}")
    return e[0] < WHOLE[dt][0] and (len(got) < 20 or e[1] < WHOLE[dt][1])


def i32(x):
    return torch.tensor(x, dtype=torch.int32, device="cuda")


# ---------------------------------------------------------------- embedding, linear epilogues, norms

@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("D", [37, 48, 1030])
@pytest.mark.parametrize("scale,buckets,mul", [(0.7, 67, (13, 5)), (1.0, 1, (1, 1)), (3.0, 1009, (2 ** 31 - 1, 2 ** 31 - 2))])
def test_embedding(K, dt, D, scale, buckets, mul):
    """Pairs over runs of several sequences, one at its first token, one going on from its slot's token, one of a single token,
    a padded row; positions; the copies that a pass's entry reads; the slots' tokens afterwards."""
    d, V, ld = DT[dt], 2000, K.act_ld(D)
    cfg = {"embedding": {"scale": scale, "bigram": {"buckets": buckets, "mul_prev": mul[0], "mul_cur": mul[1]}}}
    W = {"embed": rnd(V, D, seed=1), "bigram": rnd(buckets + 1, D, seed=2), "pos": rnd(300, D, seed=3)}
    W = {k: v.to(torch.bfloat16) for k, v in W.items()}
    Wd = {k: v.double() for k, v in W.items()}
    runs = [(0, 5, 2, 0), (5, 3, 0, 40), (8, 1, 3, 7), (9, 1, 1, 0), (10, 1, -1, 0), (11, 2, 4, 297)]    # row, rows, slot, position
    toks = S.tokens(13, V, 6)
    slots = i32([1500, 9, 8, 7, 6])
    pos = [p + e for _, n, _, p in runs for e in range(n)]
    seq = [i for i, (_, n, _, _) in enumerate(runs) for _ in range(n)]
    T = len(toks)
    nx, use = i32(toks), i32([int(t in (1, 8, 12)) for t in range(T)])            # some tokens come from the previous step
    ids = i32([0 if u else t for t, u in zip(toks, use.tolist())])
    x = torch.zeros(T, ld, device="cuda")
    cc = torch.full((T, 3 * ld), 7.0, dtype=d, device="cuda")
    K.embed(ids, W["embed"].cuda(), x, None, T, st(), prev=(nx, use), scale=scale, copies=(cc, cc[:, 2 * ld:]),
            pairs=(W["bigram"].cuda(), buckets, *mul, slots, i32(runs), i32(seq)), positions=(W["pos"].cuda(), i32(pos)))
    before = {1: 1500, 2: 7, 5: 6}
    want = torch.zeros(T, D, dtype=torch.float64)
    for i, (r0, n, slot, p) in enumerate(runs):
        if slot >= 0:
            want[r0:r0 + n] = O.embed(cfg, Wd, toks[r0:r0 + n], before.get(i), p)
    live = [t for t in range(T) if t != 10]
    assert relerr(x[live, :D], want[live]) < 1e-6
    for c in (cc[:, :D], cc[:, 2 * ld:2 * ld + D]):
        assert relerr(c[live], want[live]) < (1e-6 if dt == "f32" else 5e-3)
    assert (cc[:, D:2 * ld] == 7).all() and (cc[:, 2 * ld + D:] == 7).all()
    assert slots.tolist() == [toks[7], toks[9], toks[4], toks[8], toks[12]] and ids.tolist() == toks


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("M", [1, 20, 150, 600])
@pytest.mark.parametrize("N", [2, 50, 260])
def test_linear_epilogues(K, dt, M, N):
    """The clamped gated pair, and the decay power with an exponent per column."""
    d, Kd = DT[dt], 72
    x = rnd(M, Kd, seed=5).to(d)
    ws = [(rnd(N, Kd, seed=10 + i) / math.sqrt(Kd) * 3).to(d) for i in range(2)]
    z = [x.double() @ w.double().T for w in ws]
    bias, rate = rnd(N, seed=6, scale=4.0).float(), rnd(N, seed=7).exp().float()
    bias[0], bias[-1] = 60.0, -200.0
    P = lambda w: K.PackedLinear(w, dt == "f32", "cuda")      # noqa: E731
    gu = torch.full((M, N // 2 + 5), 7.0, dtype=d, device="cuda")
    y = torch.zeros(M, N, device="cuda")
    xa = act(x, K.act_ld(Kd), d)
    K.LinLaunch([K.Seg(P(ws[0]), xa, gu, "swiglu", ycol=2, alpha=0.9),
                 K.Seg(P(ws[1]), xa, y, "sigpow", bias=bias.cuda(), gate=rate.cuda())]).run(M, st())
    g, u = z[0][:, 0::2].clamp(max=0.9), z[0][:, 1::2].clamp(-0.9, 0.9)
    assert relerr(gu[:, 2:N // 2 + 2], g * O.sigmoid(1.702 * g) * (u + 1)) < (5e-3 if dt == "bf16" else 2e-5)
    assert (gu[:, :2] == 7).all() and (gu[:, N // 2 + 2:] == 7).all()
    want = torch.exp(-rate.double() * O.softplus(-(z[1] + bias.double())))
    assert relerr(y, want) < 2e-5 and (y[:, 0] == 1).all() and torch.isfinite(y).all()


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("D", [37, 48, 1030, 4100])
def test_norms(K, dt, D):
    """Two weights on one norm; a pass's entry, which replaces the residual; a gate on the norm; a copy of the residual."""
    d, T, eps, ld = DT[dt], 5, 1e-2, K.act_ld(D)
    tol = 1e-5 if dt == "f32" else 5e-3
    w1, w2, add = (rnd(D, seed=i).float() for i in (1, 2, 3))
    x0, y, gate = rnd(T, D, seed=4).float(), rnd(16, D, seed=5).float(), act(rnd(T, D, seed=6), ld, d)
    x = act(x0, ld, torch.float32)
    a, b = torch.zeros(T, ld, dtype=d, device="cuda"), torch.zeros(T, ld, dtype=d, device="cuda")
    cc = torch.full((T, 2 * ld), 7.0, dtype=d, device="cuda")

    def both(v):
        n = O.rms(v, eps)
        return relerr(a[:, :D], n * w1.double()) < tol and relerr(b[:, :D], n * w2.double()) < tol and (a[:, D:] == 0).all()
    K.row_norm(x, None, w1.cuda(), a, T, eps, st(), rms=True, w2=w2.cuda(), out2=b)
    assert both(x0.double())
    K.norm_add(y.cuda(), None, x, cc[:, ld:], T, eps, st(), out_norm=w1.cuda(), out=a, rms=True, slabs=2, slab_rows=8,
               out_norm2=w2.cuda(), out2=b)
    want = x0.double() + y[:T].double() + y[8:8 + T].double()
    assert both(want) and relerr(x[:, :D], want) < 1e-6 and relerr(cc[:, ld:ld + D], want) < (1e-6 if dt == "f32" else 5e-3)
    assert (cc[:, :ld] == 7).all() and (cc[:, ld + D:] == 7).all()
    K.norm_add(y.cuda(), None, x, None, T, eps, st(), out_norm=w1.cuda(), out=a, rms=True, slabs=2, slab_rows=8,
               out_norm2=w2.cuda(), out2=b, keep=False, add=add.cuda())
    want = y[:T].double() + y[8:8 + T].double() + add.double()
    assert both(want) and relerr(x[:, :D], want) < 1e-6
    K.row_norm(x, None, w1.cuda(), a, T, eps, st(), rms=True, gate=gate)
    assert relerr(a[:, :D], O.rms(want, eps) * w1.double() * gate[:, :D].double().cpu()) < tol


# ---------------------------------------------------------------- attention

@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("H,G,D,V", [(1, 1, 8, 4), (6, 2, 20, 36), (5, 5, 33, 21), (4, 2, 64, 128), (2, 1, 128, 7)])
def test_attention_rows(K, dt, H, G, D, V):
    """Queries, keys and values of their own width into the right rows, unnormed and unrotated."""
    d, T = DT[dt], 5
    Dp, _ = K.head_pad(max(D, V))
    z = rnd(T, -(-(H * D + G * D + G * V) // 4) * 4, seed=1).float().cuda()
    slot = i32([5, 0, -1, 2, 3])
    qo = torch.zeros(T, H * Dp, dtype=d, device="cuda")
    kc, vc = (torch.full((6, G * Dp), 7.0, dtype=d, device="cuda") for _ in range(2))
    K.attn_rows(z, z[:, H * D:], z[:, (H + G) * D:], None, None, None, i32([0, 1, 2, 3, 4]), slot, qo, kc, vc, T, H, G, D, Dp, 0,
                1e-5, st(), V=V)
    zc = z.cpu().to(d)
    live = [0, 1, 3, 4]
    s = slot[live].long().cpu()
    qo, kc, vc = qo.cpu().view(T, H, Dp), kc.cpu().view(6, G, Dp), vc.cpu().view(6, G, Dp)
    assert torch.equal(qo[..., :D], zc[:, :H * D].view(T, H, D)) and (qo[..., D:] == 0).all()
    assert torch.equal(kc[s][..., :D], zc[live, H * D:(H + G) * D].view(4, G, D))
    assert torch.equal(vc[s][..., :V], zc[live, (H + G) * D:(H + G) * D + G * V].view(4, G, V))
    assert (kc[..., D:] == 7).all() and (vc[..., V:] == 7).all() and (kc[[1, 4]] == 7).all() and (vc[[1, 4]] == 7).all()


def paged(d, ctxs, G, D, V, Dp, nb, bs, spikes):
    """Caches of len(ctxs) sequences in shuffled pages; spikes: per sequence [(position, key)]. Returns caches, tables, rows."""
    n = len(ctxs)
    bt = torch.randperm(n * nb, generator=torch.Generator().manual_seed(5)).view(n, nb)
    kc, vc = (torch.zeros(n * nb * bs, G, Dp, dtype=d) for _ in range(2))
    rows = []
    for t, c in enumerate(ctxs):
        k, v = rnd(c, G, D, seed=10 + t).to(d), rnd(c, G, V, seed=9000 + t).to(d)
        for at, key in spikes[t]:
            k[at] = key.to(d)
        p = torch.arange(c)
        s = bt[t][p // bs] * bs + p % bs
        kc[s, :, :D], vc[s, :, :V] = k, v
        rows.append((k.double(), v.double()))
    return kc.view(-1, G * Dp).cuda(), vc.view(-1, G * Dp).cuda(), bt.int().cuda(), rows


def loud(q, scale):
    """A key whose score with q is 9."""
    q = q.double()
    return q * 9.0 / (scale * (q @ q))


MASKS = [(37, 5), (130, 33), (1, 1), (16, 0), (64, 64), (2000, 3), (7, 40), (95, 31), (0, 0)]


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("H,G,D,V", [(6, 2, 20, 36), (5, 5, 64, 64), (33, 1, 32, 32), (4, 1, 128, 96), (3, 1, 200, 130), (4, 2, 300, 10)])
@pytest.mark.parametrize("window,keep", MASKS)
def test_decode_attention(K, dt, H, G, D, V, window, keep):
    """Contexts around page, tile, split and window edges; a key whose score stands out sits just inside or just outside the window
    or the kept tokens, or first or last; grids of several sizes (waves per workgroup), with and without splits of the keys."""
    d, bs = DT[dt], 16
    Dp, mfma = K.head_pad(max(D, V))
    mfma = mfma and dt == "bf16"
    ctxs, at = [], []
    for c in (1, 16, 33, 64, 65, 129, 300, 471):
        for p in sorted({0, c - 1, c - window, c - window - 1, keep - 1, keep} & set(range(c))):
            ctxs.append(c)
            at.append(p)
    T, scale = len(ctxs), 0.7 / math.sqrt(D)
    q = torch.zeros(T, H, Dp, dtype=d)
    q[..., :D] = rnd(T, H, D, seed=1).to(d)
    kc, vc, bt, rows = paged(d, ctxs, G, D, V, Dp, 30, bs, [[(p, loud(q[t, t % H, :D], scale))] for t, p in enumerate(at)])
    mask = {"size": window, "keep_first": keep} if window else None
    want = torch.stack([O.attend(q[t:t + 1, :, :D].double(), *rows[t], torch.tensor([c - 1]), scale, mask)[0]
                        for t, c in enumerate(ctxs)])
    wg = K.attn_groups(H, G)
    for ns, rep in ((1, 1), (3, 1), (16, 1), (1, 1 + 1024 // (T * wg))) if mfma else ((1, 1),):
        part = (torch.zeros(T * H * ns * Dp, device="cuda"), torch.zeros(T * H * ns * 2, device="cuda"),
                torch.zeros(T * wg, dtype=torch.int32, device="cuda"))
        n = T * rep
        seq, ctx = (i32(v).repeat(rep) for v in (list(range(T)), ctxs))
        out = torch.full((n + 1, H * Dp), 7.0, dtype=d, device="cuda")
        K.gqa_attention(q.view(T, -1).cuda().repeat(rep, 1), kc, vc, None, out, part, bt, bs, seq, ctx, n, H, G, Dp, mfma, ns, scale,
                        st(), window=window, keep=keep, sink=True)
        o = out[:n].view(rep, T, H, Dp).cpu()
        assert (out[n] == 7).all() and (part[2] == 0).all() and (o[..., V:] == 0).all() and (o == o[:1]).all()
        for t in range(T):
            assert relerr(o[0, t, :, :V], want[t]) < TOL[dt], (ns, rep, ctxs[t], at[t])


@pytest.mark.parametrize("dt", DT)
def test_decode_attention_far_pages(K, dt):
    """A window that lies many pages (more than a table register holds) behind the kept tokens."""
    d, bs, H, G, D, window, keep, scale = DT[dt], 16, 4, 2, 32, 200, 70, 0.2
    ctxs = [3000, 1500, 1100, 271, 270]
    at = [2800, 1299, 69, 70, 0]
    T = len(ctxs)
    q = rnd(T, H, D, seed=1).to(d)
    kc, vc, bt, rows = paged(d, ctxs, G, D, D, D, 188, bs, [[(p, loud(q[t, 0], scale))] for t, p in enumerate(at)])
    for sink, mask in ((True, {"size": window, "keep_first": keep}), (True, None)):
        for ns in (1, 4) if dt == "bf16" else (1,):
            part = (torch.zeros(T * H * ns * D, device="cuda"), torch.zeros(T * H * ns * 2, device="cuda"), i32([0] * T * G))
            out = torch.zeros(T, H * D, dtype=d, device="cuda")
            K.gqa_attention(q.view(T, -1).cuda(), kc, vc, None, out, part, bt, bs, i32(list(range(T))), i32(ctxs), T, H, G, D,
                            dt == "bf16", ns, scale, st(), window=window if mask else 0, keep=keep if mask else 0, sink=sink)
            for t in range(T):
                want = O.attend(q[t:t + 1].double(), *rows[t], torch.tensor([ctxs[t] - 1]), scale, mask)[0]
                assert relerr(out[t].view(H, D), want) < TOL[dt], (ns, t)


@pytest.mark.parametrize("H,G,D,V", [(6, 2, 20, 36), (5, 5, 64, 64), (33, 1, 32, 32), (7, 1, 128, 96), (3, 1, 200, 130)])
@pytest.mark.parametrize("waves", [4, 8])
@pytest.mark.parametrize("window,keep", MASKS)
def test_prompt_attention(K, H, G, D, V, waves, window, keep):
    """Runs of several sequences at several starts, in blocks; keys stand out for single rows just inside and outside the window
    and the kept tokens."""
    d, bs = torch.bfloat16, 16
    Dp, _ = K.head_pad(max(D, V))
    runs = [(0, 300), (130, 70), (63, 2), (0, 17), (255, 66)]       # first position, rows
    ctxs, scale = [p + n for p, n in runs], 0.7 / math.sqrt(D)
    T = sum(n for _, n in runs)
    q = torch.zeros(T, H, Dp, dtype=d)
    q[..., :D] = rnd(T, H, D, seed=1).to(d)
    row0 = [sum(n for _, n in runs[:i]) for i in range(len(runs))]
    spikes = []
    for (p, n), a in zip(runs, row0):
        s = {}
        for j, r in enumerate(sorted({0, 1, n // 3, n // 2, n - 2, n - 1} & set(range(n)))):
            i = p + r
            for at in ((i - window, keep, i), (i - window + 1, keep - 1, 0))[j % 2][:1 + j // 2]:
                if 0 <= at <= i:
                    s[at] = loud(q[a + r, j % H, :D], scale)
        spikes.append(list(s.items()))
    kc, vc, bt, rows = paged(d, ctxs, G, D, V, Dp, 21, bs, spikes)
    xmap, blocks, nx = [], [], 0
    B = 32 * waves
    for i, (p, n) in enumerate(runs):
        pos = torch.arange(p + n)
        xmap.append(bt[i].cpu()[pos // bs] * bs + pos % bs)
        blocks += [(row0[i] + o, min(B, n - o), i, p + o, nx, 0, 0, 0) for o in range(0, n, B)]
        nx += p + n
    out = torch.full((T + 1, H * Dp), 7.0, dtype=d, device="cuda")
    mask = {"size": window, "keep_first": keep} if window else None
    for sink in (True, False):
        K.gqa_prefill(q.view(T, -1).cuda(), kc, vc, torch.cat(xmap).int().cuda(), i32(blocks), len(blocks), waves, None, out, H, G,
                      Dp, scale, st(), window=window, keep=keep, sink=sink)
        o = out[:T].view(T, H, Dp).cpu()
        assert (out[T] == 7).all() and (o[..., V:] == 0).all()
        for i, (p, n) in enumerate(runs):
            k, v = rows[i]
            if not sink:                            # a plain softmax
                see = O.visible(torch.arange(p, p + n)[:, None], torch.arange(p + n)[None], mask)
                of = torch.arange(H) // (H // G)
                sc = torch.einsum("thd,khd->htk", q[row0[i]:row0[i] + n, :, :D].double(), k[:, of]) * scale
                pr = torch.softmax(sc.masked_fill(~see, -math.inf), -1)
                want = torch.einsum("htk,khd->thd", pr, v[:, of])
            else:
                want = O.attend(q[row0[i]:row0[i] + n, :, :D].double(), k, v, torch.arange(p, p + n), scale, mask)
            g = o[row0[i]:row0[i] + n, :, :V].double()
            # (rows apart: a small row's error must not hide behind a large one)
            e = (g - want).abs().amax((1, 2)) / want.abs().amax((1, 2))
            assert float(e.max()) < TOL["bf16"] * 1.5, (sink, i, int(e.argmax()))


# ---------------------------------------------------------------- the delta rule

CONV = [(1, 1, 4, 4, 1), (4, 2, 20, 28, 4), (3, 3, 33, 16, 2), (2, 1, 130, 70, 3), (2, 2, 7, 5, 6)]


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("H,G,D,V,taps", CONV)
def test_delta_conv(K, dt, H, G, D, V, taps):
    """Two sequences beside an empty run, cut at single tokens, pairs and long portions, slots dirty at the start; many rows at
    once and few."""
    d, n, nch = DT[dt], 600, 2 * G * D + H * V
    ld = nch + 3
    z, w = rnd(2, n, nch, seed=1).to(d), rnd(nch, taps, seed=2).float()
    state = torch.full((4, max(1, taps - 1) * nch), 9.0, device="cuda") if taps > 1 else None
    y, fac = torch.zeros(2, n, nch, dtype=d), torch.zeros(2, n, 2 * G)
    cuts = [0, 1, 2, 4, 5, 6, 7, 8, 10, 13, 16, 29, 30, n]
    for a, b in zip(cuts, cuts[1:]):
        m = b - a
        zz = torch.zeros(2 * m, ld, dtype=d, device="cuda")
        zz[:, :nch] = torch.cat([z[0, a:b], z[1, a:b]])
        yy, ff = torch.full((2 * m, ld), 7.0, dtype=d, device="cuda"), torch.zeros(2 * m, 2 * G, device="cuda")
        # (a single token of both: as many runs as rows)
        runs = [[0, m, 3, a], [m, m, 1, a]] + ([[0, 0, -1, 0]] if m > 1 else [])
        K.delta_conv(zz, w.cuda(), yy, ff, state, i32(runs), i32([0] * m + [1] * m), 2 * m, len(runs), H, G, D, V, st())
        assert (yy[:, nch:] == 7).all()
        y[0, a:b], y[1, a:b] = yy[:m, :nch].cpu(), yy[m:, :nch].cpu()
        fac[0, a:b], fac[1, a:b] = ff[:m].cpu(), ff[m:].cpu()
    for i, slot in ((0, 3), (1, 1)):
        want, tail = O.causal_conv(z[i].double(), w.double())
        assert relerr(y[i], O.silu(want)) < (1e-5 if dt == "f32" else 5e-3)
        if taps > 1:
            assert relerr(state[slot].view(taps - 1, nch), tail) < 1e-6
        heads = y[i, :, :2 * G * D].double().view(n, 2 * G, D)
        f = torch.rsqrt((heads * heads).sum(-1) + 1e-6)
        f[:, :G] *= D ** -0.5
        assert float((fac[i] / f - 1).abs().max()) < 1e-5
    if taps > 1:
        assert (state[0] == 9).all() and (state[2] == 9).all()


DELTA = [(1, 1, 4, 4), (4, 2, 20, 28), (2, 2, 64, 64), (2, 1, 33, 132), (1, 1, 128, 36), (3, 1, 200, 24), (2, 2, 7, 1),
         (1, 1, 256, 260)]


def delta_data(d, H, G, D, V, n):
    """Projections as the convolutions leave them, factors, decays and steps of two sequences; and as the plain scan takes them."""
    q, k, v = rnd(2, n, G * D, seed=1).to(d), rnd(2, n, G * D, seed=2).to(d), rnd(2, n, H * V, seed=3).to(d)
    k[:, 0] = q[:, 0]
    k[0, 50:54] = k[0, 49]                                  # one key again and again: corrections of what was just written
    a = torch.sigmoid(rnd(2, n, H * D, seed=4, scale=3)).float()
    a[0, 20:40, :H * D // 2] = 0.0                          # a state that is wiped out
    a[1, :, 0] = 1.0                                        # one that never decays
    beta = torch.sigmoid(rnd(2, n, H, seed=5, scale=2)).float()
    beta[0, 60:70] = 1.0
    f = [torch.rsqrt((t.double().view(2, n, G, D) ** 2).sum(-1) + 1e-6) for t in (q, k)]
    fac = torch.cat([f[0] * D ** -0.5, f[1]], -1).float()
    of = torch.arange(H) // (H // G)
    plain = [(t.double().view(2, n, G, D) * fac[..., o:o + G, None].double())[:, :, of] for t, o in ((q, 0), (k, G))]
    plain += [v.double().view(2, n, H, V), a.double().view(2, n, H, D), beta.double()]
    return (q, k, v, fac, beta, a), plain


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("H,G,D,V", DELTA)
@pytest.mark.parametrize("nseg,nt", [(1, 1), (1, 2), (2, 2), (5, 1), (16, 2)])
def test_delta_scan(K, dt, H, G, D, V, nseg, nt):
    """Two sequences in one launch beside an empty run, cut at 2, 3 and 16 tokens, slots given out of order and dirty, in
    segments: the plain recurrence however the runs are cut; with the head's norm and gate where a workgroup holds it."""
    d, n, eps = DT[dt], 330, 1e-3
    (q, k, v, fac, beta, a), plain = delta_data(d, H, G, D, V, n)
    GD, HD, HV, fused = G * D, H * D, H * V, V <= 64 * nt
    norm, g = rnd(HV, seed=7).float(), rnd(2, n, HV, seed=8).to(d)

    def run(cuts):
        S0 = torch.full((4, HD * V), 9.0, device="cuda")    # slots start dirty
        out = torch.zeros(2, n, HV)
        seg = (torch.full((3 * nseg * HD * V,), 5.0, device="cuda"), torch.full((3 * nseg * HD * D,), 5.0, device="cuda"))
        for x, y in zip((0,) + cuts, cuts + (n,)):
            m = y - x
            cat = lambda t: torch.cat([t[0, x:y], t[1, x:y]]).cuda()      # noqa: E731
            z = torch.cat([cat(q), cat(k), cat(v)], 1)
            runs = i32([[0, m, 3, x], [m, m, 1, x], [0, 0, -1, 0]])
            o = torch.zeros(2 * m, HV + 3, device="cuda")
            args = (z, z[:, GD:], z[:, 2 * GD:], cat(fac), cat(beta), cat(a), o, norm.cuda(), cat(g))
            if fused:
                y_, S1 = torch.zeros(2 * m, HV + 3, dtype=d, device="cuda"), S0.clone()
                K.delta_scan(*args, y_, S1, runs, 3, H, G, D, V, eps, (nseg, nt), seg, st())
            K.delta_scan(*args, None, S0, runs, 3, H, G, D, V, eps, (nseg, nt), seg, st())
            out[0, x:y], out[1, x:y] = o[:m, :HV].cpu(), o[m:, :HV].cpu()
            assert (o[:, HV:] == 0).all()
            if fused:
                assert torch.equal(S0, S1) and (y_[:, HV:] == 0).all()
                want = (O.rms(o[:, :HV].cpu().double().view(2 * m, H, V), eps).view(2 * m, HV) * norm.double() * cat(g).double().cpu())
                assert relerr(y_[:, :HV], want) < (2e-5 if dt == "f32" else 5e-3)
        assert (S0[0] == 9).all() and (S0[2] == 9).all()
        return out, S0
    whole, Sw = run(())
    for i, slot in ((0, 3), (1, 1)):
        want, Sx = O.delta_scan(*(t[i] for t in plain))
        assert relerr(whole[i].view(n, H, V), want) < 2e-5
        assert relerr(Sw[slot].view(H, D, V), Sx) < 2e-5
    for cuts in ((2, 4, 7, 200), (16, 32, 48, 112, 177), (15, 17, 81, 146, 329)):
        o, Sc = run(cuts)
        assert relerr(o, whole.double()) < 2e-5 and relerr(Sc, Sw.double().cpu()) < 2e-5


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("H,G,D,V", [g for g in DELTA if g[3] % 4 == 0] + [(1, 1, 16, 1024)])
def test_delta_step(K, dt, H, G, D, V):
    """Single tokens of two sequences (their first among them, a padded row between) against the plain recurrence, norm and gate."""
    d, n, eps = DT[dt], 40, 1e-3
    (q, k, v, fac, beta, a), plain = delta_data(d, H, G, D, V, 80)
    GD, HV = G * D, H * V
    norm, g = rnd(HV, seed=7).float(), rnd(2, n, HV, seed=8).to(d)
    S0 = torch.full((3, H * D * V), 9.0, device="cuda")
    want = [O.delta_scan(*(t[i][:n] for t in plain)) for i in (0, 1)]
    for t in range(n):
        cat = lambda x, e=0.0: torch.stack([x[0, t], torch.full_like(x[0, t], e), x[1, t]]).cuda()      # noqa: E731
        z = torch.cat([cat(q), cat(k), cat(v)], 1)
        out = torch.full((3, HV), 7.0, dtype=d, device="cuda")
        runs = i32([[0, 1, 2, t], [1, 0, -1, 0], [2, 1, 0, t]])
        K.delta_step(z, z[:, GD:], z[:, 2 * GD:], cat(fac), cat(beta), cat(a, 1.0), None, cat(g), None, 0, S0, runs, 3, norm.cuda(),
                     out, H, G, D, V, eps, st())
        for i, r in ((0, 0), (1, 2)):
            w = O.rms(want[i][0][t], eps).reshape(-1) * norm.double() * g[i, t].double()
            assert relerr(out[r], w) < (1e-4 if dt == "f32" else 8e-3), t
        assert (out[1] == 7).all()
    for i, s in ((0, 2), (1, 0)):
        assert relerr(S0[s].view(H, D, V), want[i][1]) < 2e-5
    assert (S0[1] == 9).all()


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("ra,rg", [(1, 3), (7, 16), (40, 64), (128, 24)])
def test_delta_step_gates(K, dt, ra, rg):
    """The step that makes its decays and gate from their low-rank inputs."""
    d, T, H, G, D, V = DT[dt], 6, 4, 2, 20, 8
    HD, HV, GD = H * D, H * V, G * D
    a2, b, low = rnd(HD, ra, seed=1).to(d) / ra ** 0.5, rnd(HD, seed=2, scale=4.0).float(), rnd(T, ra, seed=3).to(d)
    g2, lowg = rnd(HV, rg, seed=4).to(d), rnd(T, rg, seed=5).to(d)
    rate = rnd(HD, seed=6).exp().float()
    b[0], b[1] = 80.0, -150.0
    z = torch.zeros(T, 640, dtype=d, device="cuda")                   # keys are zero: the state is its decay
    z[:, 192:192 + ra], z[:, 448:448 + rg] = low, lowg
    z[:, :GD] = 1.0
    S0 = torch.ones(T, HD * V, device="cuda")
    runs = i32([[t, 1, t, 5] for t in range(T)])
    out = torch.zeros(T, HV, dtype=d, device="cuda")
    fac, beta = torch.ones(T, 2 * G, device="cuda"), torch.ones(T, H, device="cuda")
    K.delta_step(z, z[:, GD:], z[:, 2 * GD:], fac, beta, None, (z[:, 192:], a2.cuda(), b.cuda(), rate.cuda()), None,
                 (z[:, 448:], g2.cuda()), 640, S0, runs, T, torch.ones(HV, device="cuda"), out, H, G, D, V, 1e-5, st())
    want = O.sigmoid(low.double() @ a2.double().T + b.double()) ** rate.double()
    assert relerr(S0.view(T, HD, V), want[:, :, None].expand(T, HD, V)) < 1e-5
    gate = O.sigmoid(lowg.double() @ g2.double().T)
    o = O.rms(want.view(T, H, D).sum(-1, keepdim=True).expand(T, H, V), 1e-5)
    assert relerr(out, o.reshape(T, HV) * gate) < (1e-5 if dt == "f32" else 5e-3)


# ---------------------------------------------------------------- one decay per head

@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("D,V", [(4, 4), (20, 28), (64, 64), (33, 132), (7, 5), (256, 260)])
def test_lightning(K, dt, D, V):
    """Constant decays, 0 and 1 among them, over runs and segments and over single tokens: plain outputs."""
    d, n = DT[dt], 330
    decay = [0.0, 1.0, 0.5, 0.97]
    H = len(decay)
    HD, HV = H * D, H * V
    q, k, v = rnd(n, HD, seed=1).to(d) / D ** 0.5, rnd(n, HD, seed=2).to(d), rnd(n, HV, seed=3).to(d)
    a = torch.tensor(decay, device="cuda").repeat_interleave(D)[None].expand(2, -1)
    want, Sx = O.lightning_scan(*(t.double().view(n, H, -1) for t in (q, k, v)), torch.tensor(decay).double())
    zc = torch.cat([q, k, v], 1).cuda()
    zc = torch.nn.functional.pad(zc, (0, -zc.shape[1] % 8))
    for nseg, cuts in ((1, (0, n)), (5, (0, n)), (1, (0, 1, 3, 20, n)), (2, (0, 130, n)), (0, tuple(range(0, 40)) + (n,))):
        S0, out = torch.full((3, HD * V), 9.0, device="cuda"), torch.zeros(n, HV)
        seg = (torch.zeros(max(1, nseg) * HD * V, device="cuda"), torch.zeros(max(1, nseg) * HD, device="cuda"))
        for x, y in zip(cuts, cuts[1:]):
            o, z, runs = torch.zeros(y - x, HV + 4, device="cuda"), zc[x:y], i32([[0, y - x, 2, x]])
            args = (z, z[:, HD:], z[:, 2 * HD:], a)
            if y - x == 1 and V % 4 == 0:
                K.gla_step(*args, None, 1.0, S0, runs, 1, None, None, None, H, D, V, 1e-5, st(), o=o)
            else:
                K.gla_scan(*args, 1.0, o, None, None, None, S0, runs, 1, H, D, V, 1e-5, (max(1, nseg), 1 if V <= 64 else 2), seg, st())
            out[x:y] = o[:, :HV].cpu()
            assert (o[:, HV:] == 0).all()
        assert relerr(out.view(n, H, V), want) < 2e-5 and relerr(S0[2].view(H, D, V), Sx) < 2e-5, nseg
        assert (S0[:2] == 9).all()


# ---------------------------------------------------------------- one layer

@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("name,i", [(n, i) for n, c in S.CONFIGS.items() for i in range(len(c["layers"]))])
@pytest.mark.parametrize("flash", [16, 1 << 30])
def test_layer(gpu, tmp_path, dt, name, i, flash, monkeypatch):
    """One layer on given residual rows, over portions of a sequence beside a second one; prompts by blocks or row by row. Equal
    rows recur, so that a few rows hang on single far keys."""
    from nats_llm_studio_amd.models import stack
    base = S.CONFIGS[name]
    L = base["layers"][i]
    if flash != 16 and L["type"] != "attention":
        pytest.skip("no attention")
    monkeypatch.setattr(stack, "_FLASH_RUN", flash)
    cfg = {k: v for k, v in dict(base, layers=[L]).items() if k != "loop"}
    W, d, n = S.make_weights(cfg), cfg["width"], 330
    m = load(tmp_path, cfg, W, dt)
    b = m.step_buffers(512, 2, 32)
    kc, _ = m.kv_cache(64, 16)
    state = m.state_pool(3)
    for t in state.get(0, {}).values():
        t.fill_(5.0)
    x, z = rnd(n, d, seed=4), rnd(n, d, seed=9)
    for far in (0, 15, 16, 63, 64, 200, 255, 256, 270, n - 1):
        x[far] = 2 * x[5]
    blk = torch.randperm(42, generator=torch.Generator().manual_seed(1)).view(2, 21)
    layer, got = m.layers[0], {0: [], 1: []}
    from nats_llm_studio_amd.ops import stack as K
    for a, c in ((0, 1), (1, 3), (3, 67), (67, 100), (100, 300), (300, 301), (301, 330)):
        T = c - a
        for r, src in ((0, x), (1, z)):
            o = r * T
            pos = torch.arange(a, c)
            b.x[o:o + T, :d] = src[a:c].float()
            b.pos[o:o + T], b.ctx_len[o:o + T], b.tok_seq[o:o + T] = pos.int(), (pos + 1).int(), r
            b.slot[o:o + T] = (blk[r][pos // 16] * 16 + pos % 16).int()
            b.block_tables[r, :21] = blk[r].int()
            b.runs[r] = torch.tensor([o, T, 2 - r, a])
        info = m.attention_blocks(b, 2 * T)
        step = stack._Step(2 * T, 2, 16, st())
        if info:
            step.plan = m._expand_plan(b, info["qblocks"], info["row_info"], 2 * T, 16, st())
        K.row_norm(b.x, None, layer.norm1, b.h, 2 * T, cfg["norm"]["eps"], st(), rms=True, w2=layer.norm2,
                   out2=b.h2 if layer.norm2 is not None else None)
        layer.run(b, 0, kc, state.get(0), step, {})
        for r, src in ((0, x), (1, z)):
            got[r].append((b.x[r * T:(r + 1) * T, :d].cpu().double() - src[a:c].float().double()))
    Wd, eps = {k: v.double() for k, v in W.items()}, cfg["norm"]["eps"]
    for r, src in ((0, x), (1, z)):
        want, _ = O.layer(src, Wd, "l0.", L, torch.arange(n), eps)
        # (read as the residual's change)
        assert relerr(torch.cat(got[r]), want - src) < TOL[dt] * 2, r


# ---------------------------------------------------------------- whole models

@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("name", S.CONFIGS)
def test_prompt_layers(gpu, tmp_path, dt, name):
    """The residual after every layer run, and the logits, of a prompt."""
    cfg = S.CONFIGS[name]
    W, n = S.make_weights(cfg), 75
    m = load(tmp_path, cfg, W, dt)
    toks = S.tokens(n, cfg["vocab"])
    want_l = []
    want = O.forward(cfg, W, toks, layers=want_l)
    b = m.step_buffers(128, 2, 16, logit_rows=128)
    kc, _ = m.kv_cache(12, 16)
    taps = []
    orig = m.forward
    m.forward = lambda *a, **k: orig(*a, taps=taps, **k)
    (got,) = run_rows(m, b, kc, m.state_pool(2), [(1, [7, 2, 9, 4, 0], 0, toks)])
    assert len(taps) == len(want_l)
    for i, (t, w) in enumerate(zip(taps, want_l)):
        assert close(t.cpu(), w, dt), i
    assert close(got, want, dt)


def test_passes_have_their_own_states(gpu, tmp_path):
    """The runs of a looped layer share its weights; caches and states are each run's own."""
    cfg = S.CONFIGS["uneven"]
    m = load(tmp_path, cfg, S.make_weights(cfg), "bf16")
    assert m.owners == [0, 1, 2, 3, 1, 2, 3, 1, 2, 3, 4, 5] and m.layers[1] is m.layers[4] is m.layers[7]
    kc, state = m.kv_cache(4, 16)[0], m.state_pool(2)
    assert set(kc) == {2, 5, 8, 10} and set(state) == {0, 1, 3, 4, 6, 7, 9, 11, "token"}
    assert len({c[0].data_ptr() for c in kc.values()}) == 4
    assert len({s["S"].data_ptr() for k, s in state.items() if k != "token"}) == 8
    assert m.kv_token_bytes == sum(c[0][0].shape[-1] * 4 for c in kc.values())


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("name", S.CONFIGS)
def test_feed_schedules(gpu, tmp_path, dt, name):
    """One sequence whole, token by token, and in portions of several sizes; three unequal ones mixed, in reused pages and
    slots: always the plain implementation's logits."""
    cfg = S.CONFIGS[name]
    W = S.make_weights(cfg)
    m = load(tmp_path, cfg, W, dt)
    eng = engine(m)
    toks = S.tokens(150, cfg["vocab"])
    want = O.forward(cfg, W, toks)
    (whole,) = eng.feed([("w", toks, list(range(150)))])
    assert close(whole, want, dt)
    eng.feed_end("w")
    for name_, cuts in (("pairs", [2] * 20 + [1] * 10 + [100]), ("decode", [60] + [1] * 90), ("all decoded", [1] * 70 + [80]),
                        ("odd", [1, 2, 13, 16, 17, 31, 33, 37]), ("edges", [15, 1, 1, 47, 1, 63, 22])):
        assert sum(cuts) == 150
        o, rows = 0, []
        for c in cuts:
            (r,) = eng.feed([(name_, toks[o:o + c], list(range(c)))])
            rows.append(r)
            o += c
        eng.feed_end(name_)
        assert close(torch.cat(rows), want, dt), name_
    # mixed batches: (id, tokens) per step; "b" rests, "c" comes when "a" is gone
    seqs = {k: S.tokens(n, cfg["vocab"], 7 + i) for i, (k, n) in enumerate((("a", 90), ("b", 70), ("c", 120), ("d", 9)))}
    plan = [{"a": 64, "b": 1}, {"a": 2, "b": 40}, {"a": 1, "d": 5}, {"a": 1, "b": 1, "d": 1}, {"a": 1, "b": 1, "d": 1},
            {"a": 21, "b": 2, "d": 2}, {"b": 1, "c": 33}, {"b": 24, "c": 2}, {"c": 1}, {"c": 84}]
    at, got = {k: 0 for k in seqs}, {k: [] for k in seqs}
    for stp in plan:
        ent = []
        for k, n in stp.items():
            ent.append((k, seqs[k][at[k]:at[k] + n], list(range(n))))
            at[k] += n
        for (k, _, _), r in zip(ent, eng.feed(ent)):
            got[k].append(r)
        for k in stp:
            if at[k] == len(seqs[k]):
                eng.feed_end(k)
    for k, t in seqs.items():
        assert at[k] == len(t)
        assert close(torch.cat(got[k]), O.forward(cfg, W, t), dt), k
    assert eng.alloc.n_free == eng.num_blocks and len(eng.slots.free) == 4
    assert eng.counters["graph_replays"] > 20


@pytest.mark.parametrize("dt", DT)
def test_long_prompt_segments(gpu, tmp_path, dt):
    """A prompt long enough that the recurrences run in segments, alone and beside other runs, then decoded on."""
    cfg = S.CONFIGS["uneven"]
    W, n = S.make_weights(cfg), 700
    m = load(tmp_path, cfg, W, dt)
    from nats_llm_studio_amd.ops import stack as K
    assert K.gla_shape(n, 1, 3, 12)[0] > 2 and K.delta_shape(n, 1, 4, 20, 28)[0] > 2 and K.delta_shape(n - 300, 2, 4, 20, 28)[0] > 2
    eng = engine(m, ctx=1024, num_blocks=128, max_prefill_tokens=1024, max_logit_rows=1024)
    toks, other = S.tokens(n + 20, cfg["vocab"], 3), S.tokens(40, cfg["vocab"], 4)
    want = O.forward(cfg, W, toks)
    (g,) = eng.feed([("a", toks[:n], list(range(n)))])
    assert close(g, want[:n], dt)
    rows = [eng.feed([("a", [t], [0])])[0] for t in toks[n:]]
    assert close(torch.cat(rows), want[n:], dt)
    eng.feed_end("a")
    eng.feed([("b", toks[:299], [])])
    g, h = eng.feed([("b", toks[299:n], list(range(n - 299))), ("c", other, [39])])
    assert close(g, want[299:n], dt) and close(h, O.forward(cfg, W, other)[[39]], dt)


@pytest.mark.parametrize("dt", DT)
def test_batch_independence(gpu, tmp_path, dt):
    """A prompt's logits next to others, and in other pages and slots, are those it has alone, beyond rounding."""
    cfg = S.CONFIGS["uneven"]
    m = load(tmp_path, cfg, S.make_weights(cfg), dt)
    b = m.step_buffers(512, 4, 16, logit_rows=512)
    kc, _ = m.kv_cache(40, 16)
    state = m.state_pool(4)
    ps = [S.tokens(n, cfg["vocab"], n) for n in (3, 81, 130, 2)]
    blk = [[0], [3, 1, 9, 30, 31, 5], list(range(10, 19)), [39]]
    alone = [run_rows(m, b, kc, state, [(0, list(range(20, 30)), 0, p)])[0] for p in ps]
    for order in ((0, 1, 2, 3), (2, 3, 1, 0)):
        got = run_rows(m, b, kc, state, [(3 - i, blk[i], 0, ps[i]) for i in order])
        for i, g in zip(order, got):
            assert close(g, alone[i].double(), dt)


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("far,seen", [(0, (1, 1)), (19, (1, 1)), (20, (0, 0)), (209, (0, 0)), (210, (1, 0)), (248, (1, 0)),
                                      (249, (1, 1)), (360, (0, 1))])
def test_single_keys(gpu, tmp_path, dt, far, seen):
    """Two queries at places 359 and 398 with a window of 150 and 20 kept tokens: one key among hundreds, just inside or outside of
    what they see. Its exchange shows where it is seen and nowhere else, in a prompt and when decoding."""
    cfg = S.config([S.layer(S.attention(4, 2, 16, 16, 0.9, 150, 20), 0)], width=64, vocab=99, scale=1.0)
    W = S.make_weights(cfg)
    # token 97 has a direction e, token 98 a direction f that no other token has, and a query sees f as a key sees e
    e, f = torch.linalg.qr(torch.randn(64, 2, generator=torch.Generator().manual_seed(8)))[0].T
    emb = W["embed"].float()
    emb -= (emb @ e)[:, None] * e + (emb @ f)[:, None] * f
    emb[97], emb[98] = 0.2 * emb[97] + 5 * e, 0.2 * emb[98] + 5 * f
    W["embed"], W["l0.norm1"] = emb.to(torch.bfloat16), torch.ones(64, dtype=torch.bfloat16)
    W["bigram"], W["pos"] = 0 * W["bigram"], 0 * W["pos"]
    k = W["l0.mix.k"].float()
    kq = (k + torch.outer(k @ (e - f), f)).view(2, 1, 16, 64).expand(2, 2, 16, 64)
    W["l0.mix.q"] = kq.reshape(64, 64).to(torch.bfloat16)
    W["l0.mix.o"] = 3 * W["l0.mix.o"]
    m = load(tmp_path, cfg, W, dt)
    n, at = 399, [359, 398]
    toks = [t % 97 for t in S.tokens(n, 97, 3)]
    toks[at[0]] = toks[at[1]] = 98
    toks[far] = 97
    want = O.forward(cfg, W, toks)
    other = O.forward(cfg, W, toks[:far] + [5] + toks[far + 1:])
    for p, s in zip(at, seen):
        assert (S.error(want[[p]], other[[p]]) > 0.3) if s else torch.equal(want[p], other[p])
    eng = engine(m)
    (g,) = eng.feed([("p", toks, at)])
    assert close(g, want[at], dt)
    eng.feed_end("p")
    eng.feed([("q", toks[:350], [])])
    rows = [eng.feed([("q", [t], [0])])[0] for t in toks[350:]]
    assert close(torch.cat(rows), want[350:], dt)


def greedy(cfg, W, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(O.forward(cfg, W, seq)[-1].argmax()))
    return seq[len(prompt):]


@pytest.fixture(scope="module")
def expected():
    """Greedy continuations of six prompts, by the plain implementation."""
    cfg = S.CONFIGS["attention only"]
    small = S.config([S.layer(S.delta()), S.layer(S.attention()), S.layer(S.lightning(), 0)], loop=(1, 3, 2))
    out = {}
    for name, c in (("attention only", cfg), ("mixed", small)):
        W = S.make_weights(c)
        reqs = [(S.tokens(6 + 11 * i, c["vocab"], 20 + i), 24 - 2 * i) for i in range(6)]
        out[name] = c, W, reqs, [greedy(c, W, p, n) for p, n in reqs]
    return out


@pytest.mark.parametrize("name", ["attention only", "mixed"])
@pytest.mark.parametrize("blocks,graphs", [(64, True), (64, False), (7, True)])
def test_generation(gpu, tmp_path, blocks, graphs, name, expected):
    """Greedy generation of six requests over three decode rows, with and without graphs, and over a pool so small that
    sequences are preempted and prefilled again."""
    from nats_llm_studio_amd.engine.engine import GenRequest
    from nats_llm_studio_amd.engine.sampling import SamplingParams
    cfg, W, reqs, want = expected[name]
    m = load(tmp_path, cfg, W, "f32")
    eng = engine(m, max_batch=3, num_blocks=blocks, max_prefill_tokens=40, use_graphs=graphs, max_logit_rows=0)
    eng.gen_ratio = 0.0                  # admit on the prompts alone
    if graphs:
        eng.capture_all()
    futs = [eng.submit(GenRequest(p, SamplingParams(max_tokens=n, ignore_eos=True))) for p, n in reqs]
    for _ in range(1000):
        if all(f.done() for f in futs):
            break
        eng.step()
    for w, f in zip(want, futs):
        assert f.result().token_ids == w
    assert len(eng.slots.free) == 3
    assert blocks == 64 or eng.counters["preemptions"] > 0
    assert not graphs or eng.counters["graph_replays"] > 0


def test_generation_bf16(gpu, tmp_path):
    """bf16 greedy tokens are the plain implementation's, or nearly as likely; sampled ones are the same alone and in company."""
    from nats_llm_studio_amd.engine.engine import GenRequest
    from nats_llm_studio_amd.engine.sampling import SamplingParams
    cfg = S.CONFIGS["wide"]
    W = S.make_weights(cfg)
    eng = engine(load(tmp_path, cfg, W, "bf16"), max_logit_rows=0)
    p = S.tokens(60, cfg["vocab"], 5)
    r = eng.generate(p, SamplingParams(max_tokens=30, ignore_eos=True))
    lg = O.forward(cfg, W, p + r.token_ids)[len(p) - 1:-1]
    gap = lg.max(-1).values - lg[torch.arange(30), torch.tensor(r.token_ids)]
    assert float((gap / lg.std() < 0.1).double().mean()) > 0.9
    eng = engine(load(tmp_path, cfg, W, "f32"), max_logit_rows=0)
    sp = SamplingParams(max_tokens=12, ignore_eos=True, temperature=30.0, top_k=30, seed=11)
    alone = eng.generate(p, sp).token_ids
    futs = [eng.submit(GenRequest(p, sp))] + [eng.submit(GenRequest(S.tokens(9, 200, i), SamplingParams(
        max_tokens=15, ignore_eos=True))) for i in range(3)]
    while not all(f.done() for f in futs):
        eng.step()
    assert futs[0].result().token_ids == alone and len(set(alone)) > 3


def test_position_limit(gpu, tmp_path):
    """Sequences end with the learned positions."""
    from nats_llm_studio_amd.engine.sampling import SamplingParams
    cfg = dict(S.CONFIGS["ones"], max_positions=48)
    m = load(tmp_path, cfg, S.make_weights(cfg), "f32")
    assert m.cfg.ctx == 48
    r = engine(m, ctx=m.cfg.ctx, max_prefill_tokens=48, max_logit_rows=0).generate(
        S.tokens(30, cfg["vocab"]), SamplingParams(max_tokens=100, ignore_eos=True))
    assert 1 <= len(r.token_ids) <= 19 and r.finish_reason == "length"


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("name", ["ones", "odd"])
def test_long_decoding_and_graph_replays(gpu, tmp_path, dt, name):
    """A few hundred decoded tokens through the captured graph, every replay checked."""
    cfg = S.CONFIGS[name]
    W = S.make_weights(cfg)
    eng = engine(load(tmp_path, cfg, W, dt))
    toks = S.tokens(420, cfg["vocab"], 4)
    want = O.forward(cfg, W, toks)
    eng.feed([("x", toks[:20], [])])
    rows = [eng.feed([("x", [t], [0])])[0] for t in toks[20:]]
    assert close(torch.cat(rows), want[20:], dt)
    assert eng.counters["graph_replays"] > 350


def test_trace_runner(gpu, tmp_path):
    """The trace runner as a user starts it: steps on standard input, files of logits, one line per step."""
    import json
    import os
    import subprocess
    import sys
    import numpy as np
    cfg = S.CONFIGS["uneven"]
    W = S.make_weights(cfg)
    d = S.write_model(str(tmp_path / "m"), cfg, W)
    toks = S.tokens(50, cfg["vocab"], 9)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    steps = [{"step": 0, "entries": [{"id": "q", "tokens": toks[:40], "want": [39, 0]}], "end": []},
             {"step": 1, "entries": [{"id": "q", "tokens": toks[40:41], "want": []}, {"id": "r", "tokens": toks[:2], "want": [1]}],
              "end": ["r"]},
             {"step": 2, "entries": [{"id": "q", "tokens": toks[41:], "want": [8]}], "end": ["q"]}]
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", d, "--dtype", "float32", "--out",
                        str(tmp_path), "--max-tokens", "128"], input="\n".join(map(json.dumps, steps)) + "\n", text=True,
                       capture_output=True, timeout=110)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [x for x in p.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"]
    want = O.forward(cfg, W, toks)
    for n, rows in ((0, want[[39, 0]]), (1, want[[1]]), (2, want[[49]])):
        g = torch.from_numpy(np.fromfile(str(tmp_path / f"{n}.f32"), dtype="<f4")).view(-1, cfg["vocab"])
        assert g.shape == rows.shape and close(g, rows, "f32")


def test_chat_service(gpu, tmp_path):
    """A chat request over the worker's engine backend: listing, load by folder, generation, reply."""
    import threading
    from nats_llm_studio_amd.service.backends import EngineBackend
    from nats_llm_studio_amd.service.config import WorkerConfig
    from nats_llm_studio_amd.service.registry import Registry
    cfg = S.CONFIGS["uneven"]
    W = S.make_weights(cfg)
    S.write_model(str(tmp_path / "pub" / "biba"), cfg, W)
    reg = Registry(str(tmp_path))
    reg.scan()
    be = EngineBackend(WorkerConfig(models_dir=str(tmp_path), device="cuda:0", max_batch=4, max_ctx=256, dtype="float32",
                                    max_prefill_tokens=256))
    got, ev = [], threading.Event()

    def done(status, body, *a):
        got.append((status, body))
        ev.set()
    be.chat("biba", reg.resolve("biba"), {"messages": [{"role": "user", "content": "5 17 3 99"}], "max_tokens": 6,
                                          "ignore_eos": True}, done)
    assert ev.wait(100)
    status, body = got[0]
    assert status == 200, body
    assert body["model_info"]["arch"] == "Bibapel"
    assert [int(t) for t in body["choices"][0]["message"]["content"].split()] == greedy(cfg, W, [5, 17, 3, 99], 6)
    assert be.unload("biba")
