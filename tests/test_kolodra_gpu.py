"""Kolodra on the GPU kernels against the plain implementation (kolodra_oracle): each mechanism alone, then whole models
through the engine's feeds, scheduler and graphs."""
import math

import pytest
import torch

import kolodra_models as S
import kolodra_oracle as O
from stack_helpers import DT, act, engine, relerr, rnd, run_rows, st

pytestmark = pytest.mark.gpu
# Whole models: row errors (sekolorn_models.error), largest and for 19 rows of 20. The per-head norm of a few value columns
# magnifies the rounding of a row whose state output nearly cancels, hence the two bounds in bf16.
WHOLE = {"f32": (1e-5, 1e-5), "bf16": (0.1, 0.03)}
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
    return S.error(got, want) < WHOLE[dt][0] and (len(got) < 20 or S.error(got, want, 0.95) < WHOLE[dt][1])


# ---------------------------------------------------------------- linear epilogues, embedding, norms

@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("M", [1, 3, 20, 150, 600])
@pytest.mark.parametrize("N", [2, 50, 66, 260])
def test_linear_epilogues(K, dt, M, N):
    """One launch of the gated pair, the decay power, the weighted sigmoid and the softcap."""
    d, Kd = DT[dt], 72
    x = rnd(M, Kd, seed=5).to(d)
    ws = [(rnd(N, Kd, seed=10 + i) / math.sqrt(Kd) * 3).to(d) for i in range(4)]
    z = [x.double() @ w.double().T for w in ws]
    bias = rnd(N, seed=6, scale=4.0).float()
    bias[0] = 60.0                                       # no decay at all, beyond what an exponential holds
    bias[-1] = -200.0
    xa = act(x, K.act_ld(Kd), d)
    P = lambda w: K.PackedLinear(w, dt == "f32", "cuda")      # noqa: E731
    gu = torch.zeros(M, N // 2 + 5, dtype=d, device="cuda")
    gu[:, N // 2 + 2:] = 7.0
    ys = [torch.zeros(M, N, device="cuda") for _ in range(3)]
    K.LinLaunch([K.Seg(P(ws[0]), xa, gu, "geglu", ycol=2), K.Seg(P(ws[1]), xa, ys[0], "sigpow", bias=bias.cuda(), alpha=1 / 7.0),
                 K.Seg(P(ws[2]), xa, ys[1], "sigmoid", alpha=-0.6), K.Seg(P(ws[3]), xa, ys[2], "softcap", alpha=2.5)]).run(M, st())
    want = O.gelu_tanh(z[0][:, 0::2]) * z[0][:, 1::2]
    assert relerr(gu[:, 2:N // 2 + 2], want) < (5e-3 if dt == "bf16" else 2e-5)
    assert (gu[:, :2] == 0).all() and (gu[:, N // 2 + 2:] == 7).all()
    for y, w in zip(ys, [O.sigmoid(z[1] + bias.double()) ** (1 / 7.0), -0.6 * O.sigmoid(z[2]), O.softcap(z[3], 2.5)]):
        assert relerr(y, w) < 2e-5
    assert (ys[0][:, 0] == 1).all() and torch.isfinite(ys[0]).all()


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("M", [1, 5, 13, 30, 64, 100, 256, 300])
def test_split_products(K, dt, M):
    """A product whose K is split over workgroups, and the residual add over its slabs."""
    d, N, Kd, R = DT[dt], 100, 4200, 320
    w, x, res = (rnd(N, Kd, seed=1) / math.sqrt(Kd)).to(d), rnd(M, Kd, seed=2).to(d), rnd(M, N, seed=3).float()
    y = torch.full((8 * R, N), 7.0, device="cuda")
    L = K.LinLaunch([K.Seg(K.PackedLinear(w, dt == "f32", "cuda"), act(x, K.act_ld(Kd), d), y, slabs=8, slab_rows=R)])
    n = L.run(M, st())
    assert n > 1
    xr = act(res, K.act_ld(N), torch.float32)
    K.norm_add(y, None, xr, None, M, 1e-5, st(), slabs=n, slab_rows=R)
    want = x.double() @ w.double().T
    assert relerr(xr[:, :N].cpu().double() - res.double(), want) < 1e-5
    L._cfg[M] = (L.config(M), 1)                         # not split: the first slab alone
    y.fill_(7.0)
    assert L.run(M, st()) == 1 and relerr(y[:M], want) < 1e-5 and (y[R:] == 7).all()


@pytest.mark.parametrize("D", [37, 48, 1030, 4100])
def test_embed_scale_and_rms_norms(K, D):
    T, V, eps, ld = 5, 19, 1e-2, K.act_ld(D)
    tab, ids = rnd(V, D, seed=1).to(torch.bfloat16), torch.tensor([3, 0, 18, 3, 7], dtype=torch.int32)
    x, xb = torch.zeros(T, ld, device="cuda"), torch.zeros(T, ld, dtype=torch.bfloat16, device="cuda")
    K.embed(ids.cuda(), tab.cuda(), x, xb, T, st(), scale=2.3)
    want = tab.double()[ids.long()] * 2.3
    assert relerr(x[:, :D], want) < 1e-6 and relerr(xb[:, :D], want) < 5e-3
    w, y = rnd(D, seed=2).float(), rnd(T, D, seed=3).float()
    h = torch.zeros(T, ld, device="cuda")
    K.row_norm(x, None, w.cuda(), h, T, eps, st(), rms=True)
    assert relerr(h[:, :D], O.rms(want, eps) * w.double()) < 1e-5 and (h[:, D:] == 0).all()
    K.norm_add(y.cuda(), None, x, None, T, eps, st(), out_norm=w.cuda(), out=h, rms=True)
    want = want + y.double()
    assert relerr(x[:, :D], want) < 1e-6 and relerr(h[:, :D], O.rms(want, eps) * w.double()) < 1e-5
    K.norm_add(y.cuda(), None, x, None, T, eps, st())                              # the add alone
    want = want + y.double()
    K.row_norm(x, torch.tensor([4, 1], dtype=torch.int32, device="cuda"), w.cuda(), h, 2, eps, st(), rms=True)
    assert relerr(h[:2, :D], (O.rms(want, eps) * w.double())[[4, 1]]) < 1e-5


# ---------------------------------------------------------------- attention

@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("H,G,D,rot", [(1, 1, 8, 2), (6, 2, 20, 12), (5, 5, 33, 0), (40, 2, 64, 32), (8, 1, 128, 128)])
def test_attention_rows(K, dt, H, G, D, rot):
    """Norm over the whole projection, rotation of a part of each head, keys and unnormed values into the right cache rows."""
    d, T, eps = DT[dt], 7, 1e-3
    Dp, _ = K.head_pad(D)
    from nats_llm_studio_amd.ops import rope_table
    z = rnd(T, (H + G) * D, seed=1).float().cuda()
    qn, kn = rnd(H * D, seed=2).float(), rnd(G * D, seed=3).float()
    pos, slot = torch.tensor([0, 1, 300, 4, 5, 63, 64]), torch.tensor([5, 0, 9, -1, 2, 7, 3])
    cs = rope_table(512, rot, 500.0, "cuda")
    qo = torch.zeros(T, H * Dp, dtype=d, device="cuda")
    kc, vc = (torch.full((10, G * Dp), 7.0, dtype=d, device="cuda") for _ in range(2))
    K.attn_rows(z, z[:, H * D:], z[:, H * D:], qn.cuda(), kn.cuda(), cs, pos.int().cuda(), slot.int().cuda(), qo, kc, vc, T, H,
                G, D, Dp, rot, eps, st())
    W = {"q": torch.eye((H + G) * D)[:H * D].double(), "k": torch.eye((H + G) * D)[H * D:].double(), "q.norm": qn.double(),
         "k.norm": kn.double()}
    q, k, v = O.attention_rows(z.double().cpu(), W, "", {"heads": H, "kv_heads": G, "dim": D, "rot": {"base": 500.0, "dims": rot}},
                               pos, eps)
    tol = 1e-5 if dt == "f32" else 5e-3
    assert relerr(qo.view(T, H, Dp)[..., :D], q) < tol and (qo.view(T, H, Dp)[..., D:] == 0).all()
    kc, vc = kc.view(10, G, Dp), vc.view(10, G, Dp)
    live = [t for t in range(T) if slot[t] >= 0]
    assert relerr(kc[slot[live]][..., :D], k[live]) < tol and relerr(vc[slot[live]][..., :D], v[live]) < tol
    for s in (1, 4, 6, 8):
        assert (kc[s] == 7).all() and (vc[s] == 7).all()
    assert (kc[..., D:] == 7).all() and (vc[..., D:] == 7).all()


def paged(d, ctxs, G, D, Dp, nb, bs, scale, q, spikes):
    """Caches of len(ctxs) sequences in shuffled pages; a key of each whose score stands out. Returns caches, tables, rows."""
    n = len(ctxs)
    bt = torch.randperm(n * nb, generator=torch.Generator().manual_seed(5)).view(n, nb)
    kc, vc = (torch.zeros(n * nb * bs, G, Dp, dtype=d) for _ in range(2))
    rows = []
    for t, c in enumerate(ctxs):
        k, v = rnd(c, G, D, seed=10 + t).to(d), rnd(c, G, D, seed=90 + t).to(d)
        qs = q[t].double()
        k[spikes[t], :] = (qs * 9.0 / (scale * (qs @ qs))).to(d)
        p = torch.arange(c)
        s = bt[t][p // bs] * bs + p % bs
        kc[s, :, :D], vc[s, :, :D] = k, v
        rows.append((k.double(), v.double()))
    return kc.view(-1, G * Dp).cuda(), vc.view(-1, G * Dp).cuda(), bt.int().cuda(), rows


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("H,G,D", [(1, 1, 8), (6, 2, 20), (5, 5, 64), (40, 2, 64), (33, 1, 32), (8, 1, 128), (3, 1, 200), (4, 2, 300)])
def test_decode_attention(K, dt, H, G, D):
    """Contexts around the page, tile and split edges, with and without splits of the keys; a key whose score stands out sits
    at an edge, first or last; every head group's width, more than 16 heads per group included."""
    d, bs = DT[dt], 16
    Dp, mfma = K.head_pad(D)
    mfma = mfma and dt == "bf16"
    ctxs = [1, 2, 15, 16, 17, 31, 32, 33, 63, 64, 65, 127, 128, 129, 255, 256, 257, 400]
    T = len(ctxs)
    scale = 0.7 / math.sqrt(D)
    q = torch.zeros(T, H, Dp, dtype=d)
    q[..., :D] = rnd(T, H, D, seed=1).to(d)
    spikes = [min([0, c - 1, 15, 16, 31, 32, 63, 64, 255][t % 9], c - 1) for t, c in enumerate(ctxs)]
    kc, vc, bt, rows = paged(d, ctxs, G, D, Dp, 26, bs, scale, q[torch.arange(T), torch.arange(T) % H, :D], spikes)
    gate = rnd(T, H, seed=3).float()
    want = torch.stack([O.attend(q[t:t + 1, :, :D].double(), *rows[t], torch.tensor([c - 1]), scale)[0]
                        for t, c in enumerate(ctxs)]) * gate.double()[:, :, None]
    seq, ctx = torch.arange(T, dtype=torch.int32, device="cuda"), torch.tensor(ctxs, dtype=torch.int32, device="cuda")
    q, gate = q.view(T, -1).cuda(), gate.cuda()
    wg = K.attn_groups(H, G)
    for ns in (1, 3, 16) if mfma else (1,):
        part = (torch.zeros(T * H * ns * Dp, device="cuda"), torch.zeros(T * H * ns * 2, device="cuda"),
                torch.zeros(T * wg, dtype=torch.int32, device="cuda"))
        for rows_ in (T, 5):                     # grids of several sizes: one, four, eight waves per workgroup
            out = torch.full((T, H * Dp), 7.0, dtype=d, device="cuda")
            K.gqa_attention(q, kc, vc, gate, out, part, bt, bs, seq, ctx, rows_, H, G, Dp, mfma, ns, scale, st())
            o = out.view(T, H, Dp)
            for t in range(rows_):
                assert relerr(o[t, :, :D], want[t]) < TOL[dt], (ns, ctxs[t])
            assert (o[:rows_, :, D:] == 0).all() and (o[rows_:] == 7).all() and (part[2] == 0).all()
    ctx[3] = 0                                   # a padded row (no keys) leaves zeros
    K.gqa_attention(q, kc, vc, gate, out, part, bt, bs, seq, ctx, T, H, G, Dp, mfma, 1, scale, st())
    assert (out[3] == 0).all()


@pytest.mark.parametrize("H,G,D", [(1, 1, 20), (6, 2, 32), (5, 5, 64), (40, 2, 64), (33, 1, 32), (7, 1, 128), (12, 4, 100), (3, 1, 200)])
@pytest.mark.parametrize("waves", [4, 8])
def test_prompt_attention(K, H, G, D, waves):
    """Runs of several sequences at several starts, in blocks; each row's own key stands out for some rows, an early, a tile's
    edge or a later (unseen) one for others."""
    d, bs = torch.bfloat16, 16
    Dp, _ = K.head_pad(D)
    runs = [(0, 300), (130, 70), (63, 2), (64, 1), (0, 17), (255, 66)]       # first position, rows
    ctxs, scale = [p + n for p, n in runs], 0.7 / math.sqrt(D)
    T = sum(n for _, n in runs)
    q = torch.zeros(T, H, Dp, dtype=d)
    q[..., :D] = rnd(T, H, D, seed=1).to(d)
    row0 = [sum(n for _, n in runs[:i]) for i in range(len(runs))]
    last = [a + n - 1 for a, (_, n) in zip(row0, runs)]
    spikes = [0, 64, 63, 64, 16, 256]
    kc, vc, bt, rows = paged(d, ctxs, G, D, Dp, 21, bs, scale, q[last, 0, :D], spikes)
    gate = rnd(T, H, seed=3).float()
    xmap, blocks, nx = [], [], 0
    B = 32 * waves
    for i, (p, n) in enumerate(runs):
        pos = torch.arange(p + n)
        xmap.append(bt[i].cpu()[pos // bs] * bs + pos % bs)
        blocks += [(row0[i] + o, min(B, n - o), i, p + o, nx, 0, 0, 0) for o in range(0, n, B)]
        nx += p + n
    out = torch.full((T + 1, H * Dp), 7.0, dtype=d, device="cuda")
    K.gqa_prefill(q.view(T, -1).cuda(), kc, vc, torch.cat(xmap).int().cuda(), torch.tensor(blocks, dtype=torch.int32).cuda(),
                  len(blocks), waves, gate.cuda(), out, H, G, Dp, scale, st())
    assert (out[T] == 7).all()
    o = out[:T].view(T, H, Dp)
    assert (o[..., D:] == 0).all()
    for i, (p, n) in enumerate(runs):
        s = slice(row0[i], row0[i] + n)
        want = O.attend(q[s, :, :D].double(), *rows[i], torch.arange(p, p + n), scale) * gate[s].double()[:, :, None]
        for r in range(n):                       # (rows apart: a small row's error must not hide behind a large one)
            assert relerr(o[s][r, :, :D], want[r]) < TOL["bf16"] * 1.5, (i, r)


# ---------------------------------------------------------------- the recurrence

GLA = [(1, 4, 4), (3, 20, 28), (2, 64, 64), (2, 33, 132), (1, 128, 36), (1, 200, 24), (2, 7, 1), (1, 256, 260)]


def gla_data(d, H, D, V, n):
    q, k, v = rnd(2, n, H * D, seed=1).to(d), rnd(2, n, H * D, seed=2).to(d), rnd(2, n, H * V, seed=3).to(d)
    k[:, 0] = q[:, 0]                                       # (no first output that nearly cancels and is then normed)
    a = torch.sigmoid(rnd(2, n, H * D, seed=4, scale=3)).float()
    a[0, 20:40, :H * D // 2] = 0.0                          # a state that is wiped out
    a[1, :, 0] = 1.0                                        # one that never decays
    return q, k, v, a


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("H,D,V", GLA)
@pytest.mark.parametrize("nseg,nt", [(1, 1), (1, 2), (2, 2), (5, 1), (16, 2)])
def test_gla_scan(K, dt, H, D, V, nseg, nt):
    """Two sequences in one launch beside an empty run, cut at 2, 3 and 16 tokens, slots given out of order and dirty, in
    segments: the plain recurrence however the runs are cut; with the head's norm and gate where a workgroup holds it."""
    d, n, qs, eps = DT[dt], 330, 0.37, 1e-3
    q, k, v, a = gla_data(d, H, D, V, n)
    HD, HV, fused = H * D, H * V, V <= 64 * nt
    norm, g = rnd(HV, seed=7).float(), rnd(2, n, HV, seed=8).to(d)

    def run(cuts):
        S0 = torch.full((4, HD * V), 9.0, device="cuda")    # slots start dirty
        out = torch.zeros(2, n, HV)
        seg = (torch.full((3 * nseg * HD * V,), 5.0, device="cuda"), torch.full((3 * nseg * HD,), 5.0, device="cuda"))
        for x, y in zip((0,) + cuts, cuts + (n,)):
            m = y - x
            cat = lambda t: torch.cat([t[0, x:y], t[1, x:y]])      # noqa: E731
            z = torch.cat([cat(q), cat(k), cat(v)], 1).cuda()
            runs = torch.tensor([[0, m, 3, x], [m, m, 1, x], [0, 0, -1, 0]], dtype=torch.int32, device="cuda")
            o = torch.zeros(2 * m, HV + 3, device="cuda")
            args = (z, z[:, HD:], z[:, 2 * HD:], cat(a).cuda(), qs, o, norm.cuda(), cat(g).cuda())
            if fused:
                y_, S1 = torch.zeros(2 * m, HV + 3, dtype=d, device="cuda"), S0.clone()
                K.gla_scan(*args, y_, S1, runs, 3, H, D, V, eps, (nseg, nt), seg, st())
            K.gla_scan(*args, None, S0, runs, 3, H, D, V, eps, (nseg, nt), seg, st())
            out[0, x:y], out[1, x:y] = o[:m, :HV].cpu(), o[m:, :HV].cpu()
            assert (o[:, HV:] == 0).all()
            if fused:
                assert torch.equal(S0, S1) and (y_[:, HV:] == 0).all()
                want = (O.rms(o[:, :HV].cpu().double().view(2 * m, H, V), eps).view(2 * m, HV) * norm.double() * cat(g).double())
                assert relerr(y_[:, :HV], want) < (2e-5 if dt == "f32" else 5e-3)
        assert (S0[0] == 9).all() and (S0[2] == 9).all()
        return out, S0
    whole, Sw = run(())
    for i, slot in ((0, 3), (1, 1)):
        want, Sx = O.gla_scan(*(t[i].double().view(n, H, -1) for t in (q, k, v, a)))
        assert relerr(whole[i].view(n, H, V), want * qs) < 2e-5
        assert relerr(Sw[slot].view(H, D, V), Sx) < 2e-5
    for cuts in ((2, 4, 7, 200), (16, 32, 48, 112, 177), (15, 17, 81, 146, 329)):
        o, Sc = run(cuts)
        assert relerr(o, whole.double()) < 2e-5 and relerr(Sc, Sw.double().cpu()) < 2e-5


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("H,D,V", [g for g in GLA if g[2] % 4 == 0] + [(1, 16, 1024)])
def test_gla_step(K, dt, H, D, V):
    """Single tokens of two sequences (one slot's first token among them, a padded row between) against the scan and its
    output norm."""
    d, n, qs, eps = DT[dt], 40, 0.37, 1e-3
    q, k, v, a = gla_data(d, H, D, V, n)
    HD, HV = H * D, H * V
    norm, g = rnd(HV, seed=7).float().cuda(), rnd(2, n, HV, seed=8).to(d)
    z = torch.cat([torch.cat([q[i], k[i], v[i]], 1) for i in (0, 1)]).cuda()
    o, want = torch.zeros(2 * n, HV, device="cuda"), torch.zeros(2 * n, HV, dtype=d, device="cuda")
    Sw = torch.full((3, HD * V), 9.0, device="cuda")
    runs = torch.tensor([[0, n, 2, 0], [n, n, 0, 0]], dtype=torch.int32, device="cuda")
    K.gla_scan(z, z[:, HD:], z[:, 2 * HD:], a.view(2 * n, HD).cuda(), qs, o, None, None, None, Sw, runs, 2, H, D, V, eps, (1, 1),
               None, st())
    K.scan_out(o, norm, g.view(2 * n, HV).cuda(), want, H, V, 2 * n, eps, st())
    ref = O.rms(o.double().cpu().view(2 * n, H, V), eps).view(2 * n, HV) * norm.double().cpu() * g.double().view(2 * n, HV)
    assert relerr(want, ref) < (1e-5 if dt == "f32" else 5e-3)
    S0 = torch.full((3, HD * V), 9.0, device="cuda")
    for t in range(n):
        zz = torch.stack([z[t], torch.zeros_like(z[t]), z[n + t]])
        aa = torch.stack([a[0, t], a[0, t], a[1, t]]).cuda()
        gg = torch.stack([g[0, t], g[0, t], g[1, t]]).cuda()
        out = torch.full((3, HV), 7.0, dtype=d, device="cuda")
        runs = torch.tensor([[0, 1, 2, t], [1, 0, -1, 0], [2, 1, 0, t]], dtype=torch.int32, device="cuda")
        K.gla_step(zz, zz[:, HD:], zz[:, 2 * HD:], aa, None, qs, S0, runs, 3, norm, gg, out, H, D, V, eps, st())
        assert relerr(out[[0, 2]], want[[t, n + t]].double().cpu()) < (3e-5 if dt == "f32" else 8e-3)
        assert (out[1] == 7).all()
    assert relerr(S0[[0, 2]], Sw[[0, 2]].double().cpu()) < 1e-6 and (S0[1] == 9).all()


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("R", [1, 7, 16, 40])
def test_gla_step_decays(K, dt, R):
    """The step that makes its own decays from the low-rank gate input: the state they leave."""
    d, T, H, D, V = DT[dt], 6, 3, 20, 8
    HD = H * D
    a2, b, low = rnd(HD, R, seed=1).to(d), rnd(HD, seed=2, scale=4.0).float(), rnd(T, R, seed=3).to(d)
    b[0], b[1] = 80.0, -150.0
    z = torch.zeros(T, 256, dtype=d, device="cuda")                   # keys are zero: the state is its decay
    z[:, 192:192 + R] = low
    S0 = torch.ones(T, HD * V, device="cuda")
    runs = torch.tensor([[t, 1, t, 5] for t in range(T)], dtype=torch.int32, device="cuda")
    out = torch.zeros(T, H * V, dtype=d, device="cuda")
    K.gla_step(z, z[:, HD:], z[:, 2 * HD:], None, (z[:, 192:], a2.cuda(), b.cuda(), 1 / 5.0), 1.0, S0, runs, T,
               torch.ones(H * V, device="cuda"), torch.ones(T, H * V, dtype=d, device="cuda"), out, H, D, V, 1e-5, st())
    want = O.sigmoid(low.double() @ a2.double().T + b.double()) ** (1 / 5.0)
    assert relerr(S0.view(T, HD, V), want[:, :, None].expand(T, HD, V)) < 1e-5


# ---------------------------------------------------------------- one layer

@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("name,i", [("uneven", 0), ("uneven", 1), ("uneven", 3), ("ones", 0), ("wide", 0), ("wide", 1),
                                    ("big heads", 0), ("big heads", 1), ("odd", 0), ("odd", 1)])
@pytest.mark.parametrize("flash", [16, 1 << 30])
def test_layer(gpu, tmp_path, dt, name, i, flash, monkeypatch):
    """One layer on given residual rows, over portions of a sequence beside a second one; prompts by blocks or row by row. One
    direction is boosted so that a few rows hang on single far keys."""
    from nats_llm_studio_amd.models import stack
    monkeypatch.setattr(stack, "_FLASH_RUN", flash)
    base = S.CONFIGS[name]
    cfg = dict(base, layers=[{k: v for k, v in base["layers"][i].items() if k != "weights_of"}])
    W, d, n = S.make_weights(cfg), cfg["width"], 330
    m = load(tmp_path, cfg, W, dt)
    b = m.step_buffers(512, 2, 32)
    kc, _ = m.kv_cache(64, 16)
    state = m.state_pool(3)
    for t in state[0].values():
        t.fill_(5.0)
    x, z = rnd(n, d, seed=4), rnd(n, d, seed=9)
    for far in (0, 15, 16, 63, 64, 200, 255, 256, 270, n - 1):          # equal rows: queries and keys agree but for the rotation
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
        assert bool(info) == (dt == "bf16" and T >= flash and K.head_pad(cfg["layers"][0]["mixer"]["left"]["dim"])[1])
        step = stack._Step(2 * T, 2, 16, st())
        if info:
            step.plan = m._expand_plan(b, info["qblocks"], info["row_info"], 2 * T, 16, st())
        K.row_norm(b.x, None, layer.norm1, b.h, 2 * T, cfg["norm"]["eps"], st(), rms=True)
        layer.run(b, 0, kc, state[0], step, {})
        for r, src in ((0, x), (1, z)):
            got[r].append((b.x[r * T:(r + 1) * T, :d].cpu().double() - src[a:c].float().double()))
    Wd, eps, L = {k: v.double() for k, v in W.items()}, cfg["norm"]["eps"], cfg["layers"][0]
    for r, src in ((0, x), (1, z)):
        h = O.norm_one_plus(src, Wd["l0.norm1"], eps)
        want, _ = O.parallel_mixer(h, Wd, "l0.mix.", L["mixer"], torch.arange(n), eps)
        if L["mlp"]:
            want = want + O.dense_ff(h, Wd, "l0.mlp.")
        # (read as the residual's change)
        assert relerr(torch.cat(got[r]), want) < TOL[dt] * 2, r


# ---------------------------------------------------------------- whole models

@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("name", S.CONFIGS)
def test_prompt_layers(gpu, tmp_path, dt, name):
    """The residual after every layer, and the logits, of a prompt."""
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
    for t, w in zip(taps, want_l):
        assert close(t.cpu(), w, dt)
    assert close(got, want, dt)


def test_shared_weights(gpu, tmp_path):
    """Layers with another's weights share its tensors and have caches and states of their own."""
    cfg = S.CONFIGS["uneven"]
    m = load(tmp_path, cfg, S.make_weights(cfg), "bf16")
    assert m.layers[2] is m.layers[0] and m.layers[5] is m.layers[0] and m.layers[4] is m.layers[1]
    kc, state = m.kv_cache(4, 16)[0], m.state_pool(2)
    assert set(kc) == set(state) == set(range(6))
    assert len({c[0].data_ptr() for c in kc.values()}) == 6 and len({s["S"].data_ptr() for s in state.values()}) == 6
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
    """A prompt long enough that the recurrence runs in segments, alone and beside other runs, then decoded on."""
    cfg = S.CONFIGS["uneven"]
    W, n = S.make_weights(cfg), 700
    m = load(tmp_path, cfg, W, dt)
    from nats_llm_studio_amd.ops import stack as K
    assert K.gla_shape(n, 1, 3, 28)[0] > 2 and K.gla_shape(n - 300, 2, 3, 28)[0] > 2
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
@pytest.mark.parametrize("far", [0, 17, 31, 32])
def test_far_key(gpu, tmp_path, dt, far):
    """Attention finds one early key among hundreds: its exchange shows, in a prompt and when decoding."""
    a = S.left(4, 2, 16, 0, 1.0, 0.9)
    cfg = S.config([S.layer(a, S.right(1, 4, 4, 1.0), 0, 2.0, 0.1)], width=64, vocab=99)
    W = S.make_weights(cfg)
    # no rotation; token 97 has a direction e, token 98 a direction f that no other token has, and a query sees f as a key
    # sees e
    e, f = torch.linalg.qr(torch.randn(64, 2, generator=torch.Generator().manual_seed(8)))[0].T
    emb = W["embed"].float()
    emb -= (emb @ e)[:, None] * e + (emb @ f)[:, None] * f
    emb[97], emb[98] = 0.2 * emb[97] + 5 * e, 0.2 * emb[98] + 5 * f
    W["embed"], W["l0.norm1"] = emb.to(torch.bfloat16), torch.zeros(64, dtype=torch.bfloat16)
    k = W["l0.mix.left.k"].float()
    kq = (k + torch.outer(k @ (e - f), f)).view(2, 1, 16, 64).expand(2, 2, 16, 64)
    W["l0.mix.left.q"] = kq.reshape(64, 64).to(torch.bfloat16)
    for w, h in (("q", 4), ("k", 2)):
        W[f"l0.mix.left.{w}.norm"] = torch.full((h * 16,), 1.3, dtype=torch.bfloat16)
    m = load(tmp_path, cfg, W, dt)
    n = 400
    toks = [t % 97 for t in S.tokens(n, 97, 3)]
    toks[far], toks[-1], toks[-40] = 97, 98, 98
    want = O.forward(cfg, W, toks)
    other = O.forward(cfg, W, toks[:far] + [5] + toks[far + 1:])
    assert S.error(want[[n - 40]], other[[n - 40]]) > 0.3
    eng = engine(m)
    (g,) = eng.feed([("p", toks, [n - 40, n - 1])])
    assert close(g, want[[n - 40, n - 1]], dt)
    eng.feed_end("p")
    eng.feed([("q", toks[:n - 40], [])])
    rows = [eng.feed([("q", [t], [0])])[0] for t in toks[n - 40:]]
    assert close(torch.cat(rows), want[n - 40:], dt)


def greedy(cfg, W, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(O.forward(cfg, W, seq)[-1].argmax()))
    return seq[len(prompt):]


@pytest.mark.parametrize("blocks,graphs", [(64, True), (64, False), (7, True)])
def test_generation(gpu, tmp_path, blocks, graphs):
    """Greedy generation of six requests over three decode rows, with and without graphs, and over a pool so small that
    sequences are preempted and prefilled again."""
    from nats_llm_studio_amd.engine.engine import GenRequest
    from nats_llm_studio_amd.engine.sampling import SamplingParams
    cfg = S.CONFIGS["uneven"]
    W = S.make_weights(cfg)
    m = load(tmp_path, cfg, W, "f32")
    eng = engine(m, max_batch=3, num_blocks=blocks, max_prefill_tokens=40, use_graphs=graphs, max_logit_rows=0)
    eng.gen_ratio = 0.0                  # admit on the prompts alone
    if graphs:
        eng.capture_all()
    reqs = [(S.tokens(6 + 11 * i, cfg["vocab"], 20 + i), 24 - 2 * i) for i in range(6)]
    futs = [eng.submit(GenRequest(p, SamplingParams(max_tokens=n, ignore_eos=True))) for p, n in reqs]
    for _ in range(1000):
        if all(f.done() for f in futs):
            break
        eng.step()
    for (p, n), f in zip(reqs, futs):
        assert f.result().token_ids == greedy(cfg, W, p, n)
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
    sp = SamplingParams(max_tokens=12, ignore_eos=True, temperature=0.9, top_k=30, seed=11)
    alone = eng.generate(p, sp).token_ids
    futs = [eng.submit(GenRequest(p, sp))] + [eng.submit(GenRequest(S.tokens(9, 200, i), SamplingParams(
        max_tokens=15, ignore_eos=True))) for i in range(3)]
    while not all(f.done() for f in futs):
        eng.step()
    assert futs[0].result().token_ids == alone and len(set(alone)) > 3


@pytest.mark.parametrize("dt", DT)
def test_long_decoding_and_graph_replays(gpu, tmp_path, dt):
    """A few hundred decoded tokens through the captured graph, every replay checked."""
    cfg = S.CONFIGS["ones"]
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
    S.write_model(str(tmp_path / "pub" / "kolo"), cfg, W)
    reg = Registry(str(tmp_path))
    reg.scan()
    be = EngineBackend(WorkerConfig(models_dir=str(tmp_path), device="cuda:0", max_batch=4, max_ctx=256, dtype="float32",
                                    max_prefill_tokens=256))
    got, ev = [], threading.Event()

    def done(status, body, *a):
        got.append((status, body))
        ev.set()
    be.chat("kolo", reg.resolve("kolo"), {"messages": [{"role": "user", "content": "5 17 3 99"}], "max_tokens": 6,
                                          "ignore_eos": True}, done)
    assert ev.wait(100)
    status, body = got[0]
    assert status == 200, body
    assert body["model_info"]["arch"] == "Kolodra"
    assert [int(t) for t in body["choices"][0]["message"]["content"].split()] == greedy(cfg, W, [5, 17, 3, 99], 6)
    assert be.unload("kolo")
