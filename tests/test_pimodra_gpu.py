"""Pimodra on the GPU kernels against the plain implementation (pimodra_oracle): each mechanism alone, then whole models
through the engine's feeds, scheduler and graphs."""
import math

import pytest
import torch

import pimodra_models as S
import pimodra_oracle as O
from stack_helpers import DT, act, engine, relerr, rnd, run_rows, st

pytestmark = pytest.mark.gpu
# Whole models: row errors (sekolorn_models.error), largest and for 19 rows of 20. Group norms magnify the rounding of a row whose
# part of a sublayer's output nearly cancels ahead of them, hence the two bounds in bf16.
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


# ---------------------------------------------------------------- attention

SHAPES = [(6, 2, 20, 36), (5, 5, 64, 64), (32, 1, 32, 32), (7, 1, 128, 96), (32, 8, 128, 128), (20, 10, 64, 50), (9, 3, 128, 128),
          (1, 1, 8, 8), (24, 24, 96, 128)]
PLAIN = [(3, 1, 200, 130), (40, 4, 32, 32), (70, 10, 64, 20), (4, 2, 300, 10), (2, 2, 260, 260)]
WINDOWS = [37, 130, 1, 16, 33, 64, 2000, 95, 0]


def paged(d, ctxs, G, D, V, Dp, nb, bs, spikes):
    """Caches of len(ctxs) sequences in shuffled pages; spikes: per sequence [(position, key head, key)]. Returns caches, tables,
    rows."""
    n = len(ctxs)
    bt = torch.randperm(n * nb, generator=torch.Generator().manual_seed(5)).view(n, nb)
    kc, vc = (torch.zeros(n * nb * bs, G, Dp, dtype=d) for _ in range(2))
    rows = []
    for t, c in enumerate(ctxs):
        k, v = rnd(c, G, D, seed=10 + t).to(d), rnd(c, G, V, seed=9000 + t).to(d)
        for at, g, key in spikes[t]:
            k[at, g] = key.to(d)
        p = torch.arange(c)
        s = bt[t][p // bs] * bs + p % bs
        kc[s, :, :D], vc[s, :, :V] = k, v
        rows.append((k.double(), v.double()))
    return kc.view(-1, G * Dp).cuda(), vc.view(-1, G * Dp).cuda(), bt.int().cuda(), rows


def key_tiles(kc, G):
    """Rows of keys [slots][G * Dp] as tiles of 16 slots."""
    return kc.view(kc.shape[0] // 16, 16, G, -1, 8).permute(0, 2, 3, 1, 4).reshape(kc.shape)


def key_rows(kc, G):
    return kc.view(kc.shape[0] // 16, G, -1, 16, 8).permute(0, 3, 1, 2, 4).reshape(kc.shape)


def loud(q, scale):
    """A key whose score with q is 9."""
    q = q.double()
    return q * 9.0 / (scale * (q @ q))


def talk_inputs(d, T, H, D, V, Dp, seed=1):
    q = torch.zeros(T, H, Dp, dtype=d)
    q[..., :D] = rnd(T, H, D, seed=seed).to(d)
    talk = (rnd(H, H, seed=seed + 1) / math.sqrt(H) + torch.eye(H)).to(torch.bfloat16)
    gate = torch.sigmoid(rnd(T, H * V, seed=seed + 2)).to(d)
    return q, talk, gate


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("H,G,D,V", SHAPES + PLAIN)
@pytest.mark.parametrize("window", WINDOWS)
def test_decode_attention(K, dt, H, G, D, V, window):
    """Contexts around page, tile, split and window edges; a key whose score stands out sits just inside or just outside the window,
    or first or last; grids of several sizes, with and without splits of the keys, in one launch and in several."""
    d, bs = DT[dt], 16
    Dp, _ = K.head_pad(max(D, V))
    ctxs, at = [], []
    for c in (1, 16, 33, 64, 65, 129, 300, 471):
        for p in sorted({0, c - 1, c - window, c - window - 1} & set(range(c))):
            ctxs.append(c)
            at.append(p)
    T, scale = len(ctxs), 0.7 / math.sqrt(D)
    q, talk, gate = talk_inputs(d, T, H, D, V, Dp)
    spikes = [[(p, t % H // (H // G), loud(q[t, t % H, :D], scale))] for t, p in enumerate(at)]
    kc, vc, bt, rows = paged(d, ctxs, G, D, V, Dp, 30, bs, spikes)
    mask = {"size": window} if window else None
    want = torch.stack([O.attend(q[t:t + 1, :, :D].double(), *rows[t], torch.tensor([c - 1]), scale, mask, talk.double())[0]
                        for t, c in enumerate(ctxs)]) * gate.double().view(T, H, V)
    plan = K.TalkPlan(H, G, Dp, window, 480, dt == "f32", "cuda")
    assert plan.mfma == (dt == "bf16" and Dp <= 256)
    if plan.mfma:
        kc = key_tiles(kc, G)
    m = plan.matrix(talk)
    ld = H * V + 5
    for rep, rows_at_once in ((1, None), (1, 7), (1 + 1024 // (T * plan.groups), None)) if plan.mfma else ((1, None),):
        n = T * rep
        seq, ctx = (i32(v).repeat(rep) for v in (list(range(T)), ctxs))
        g = torch.zeros(n, ld, dtype=d, device="cuda")
        g[:, :H * V] = gate.cuda().repeat(rep, 1)
        out = torch.full((n + 1, H * Dp), 7.0, dtype=d, device="cuda")
        plan.rows = lambda cap, most=rows_at_once or n: min(cap, most)
        sizes = plan.scratch(n) if plan.mfma else ()
        part = [torch.full((s,), math.nan, device="cuda") for s in sizes[:3]] + [
            torch.zeros(s, dtype=torch.int32, device="cuda") for s in sizes[3:]]
        for again in range(2):
            K.talk_attention(plan, q.view(T, -1).cuda().repeat(rep, 1), kc, vc, m, g, out, part, bt, bs, seq, ctx, n, V, scale, st())
        o = out[:n].view(rep, T, H, Dp).cpu()
        assert (out[n] == 7).all() and (o[..., V:] == 7).all() and (o == o[:1]).all()
        assert not part or (part[3] == 0).all()
        for t in range(T):
            assert relerr(o[0, t, :, :V], want[t]) < TOL[dt], (rep, rows_at_once, ctxs[t], at[t])


@pytest.mark.parametrize("H,G,D,V", SHAPES)
@pytest.mark.parametrize("waves", [4, 8])
@pytest.mark.parametrize("window", WINDOWS)
def test_prompt_attention(K, H, G, D, V, waves, window):
    """Runs of several sequences at several starts, in blocks; keys stand out for single rows just inside and outside the window."""
    d, bs = torch.bfloat16, 16
    Dp, _ = K.head_pad(max(D, V))
    runs = [(0, 300), (130, 70), (63, 2), (0, 17), (255, 66)]       # first position, rows
    ctxs, scale = [p + n for p, n in runs], 0.7 / math.sqrt(D)
    T = sum(n for _, n in runs)
    q, talk, gate = talk_inputs(d, T, H, D, V, Dp)
    row0 = [sum(n for _, n in runs[:i]) for i in range(len(runs))]
    spikes = []
    for (p, n), a in zip(runs, row0):
        s = []
        for j, r in enumerate(sorted({0, 1, n // 3, n // 2, n - 2, n - 1} & set(range(n)))):
            i, h = p + r, j % H
            for at in ((i - window, i), (i - window + 1, 0))[j % 2]:
                if 0 <= at <= i:
                    s.append((at, h // (H // G), loud(q[a + r, h, :D], scale)))
        spikes.append(s)
    kc, vc, bt, rows = paged(d, ctxs, G, D, V, Dp, 21, bs, spikes)
    B = 32 * waves
    blocks = [(row0[i] + o, min(B, n - o), i, p + o, 0, 0, 0, 0) for i, (p, n) in enumerate(runs) for o in range(0, n, B)]
    out = torch.full((T + 1, H * Dp), 7.0, dtype=d, device="cuda")
    mask = {"size": window} if window else None
    plan = K.TalkPlan(H, G, Dp, window, 480, False, "cuda")
    assert plan.prefill
    K.talk_prefill(plan, q.view(T, -1).cuda(), key_tiles(kc, G), vc, plan.matrix(talk), gate.cuda(), out, bt, bs, i32(blocks), len(blocks), waves, V,
                   scale, st())
    o = out[:T].view(T, H, Dp).cpu()
    assert (out[T] == 7).all() and (o[..., V:] == 7).all()
    for i, (p, n) in enumerate(runs):
        w = O.attend(q[row0[i]:row0[i] + n, :, :D].double(), *rows[i], torch.arange(p, p + n), scale, mask, talk.double())
        want = w * gate[row0[i]:row0[i] + n].double().view(n, H, V)
        g = o[row0[i]:row0[i] + n, :, :V].double()
        # (rows apart: a small row's error must not hide behind a large one)
        e = (g - want).abs().amax((1, 2)) / want.abs().amax((1, 2))
        assert float(e.max()) < TOL["bf16"] * 1.5, (i, int(e.argmax()))


@pytest.mark.parametrize("dt", DT)
def test_attention_far_pages(K, dt):
    """Contexts of more pages than a table register holds, seen whole or through a window, decoded and as the end of a prompt."""
    d, bs, H, G, D, scale = DT[dt], 16, 4, 2, 32, 0.2
    ctxs, at = [3000, 1500, 1100, 271], [2801, 0, 900, 72]
    T = len(ctxs)
    q, talk, gate = talk_inputs(d, 16 * T, H, D, D, D)
    spikes = [[(p, 0, loud(q[16 * t + 15, 0], scale))] for t, p in enumerate(at)]
    kc, vc, bt, rows = paged(d, ctxs, G, D, D, D, 188, bs, spikes)
    for window in (200, 0):
        plan = K.TalkPlan(H, G, D, window, 3008, dt == "f32", "cuda")
        m, mask = plan.matrix(talk), {"size": window} if window else None
        last = torch.arange(T) * 16 + 15
        want = torch.cat([O.attend(q[16 * t:16 * t + 16].double(), *rows[t], torch.arange(c - 16, c), scale, mask, talk.double())
                          for t, c in enumerate(ctxs)]) * gate.double().view(-1, H, D)
        part = [torch.zeros(s, device="cuda") for s in plan.scratch(T)[:3]] + [i32([0] * T * G)] if plan.mfma else ()
        keys = key_tiles(kc, G) if plan.mfma else kc
        out = torch.zeros(16 * T, H * D, dtype=d, device="cuda")
        K.talk_attention(plan, q[last].reshape(T, -1).cuda(), keys, vc, m, gate[last].cuda(), out, part, bt, bs, i32(list(range(T))),
                         i32(ctxs), T, D, scale, st())
        for t in range(T):
            assert relerr(out[t].view(H, D), want[last[t]]) < TOL[dt], (window, t)
        if plan.prefill:
            blocks = i32([(16 * t, 16, t, c - 16, 0, 0, 0, 0) for t, c in enumerate(ctxs)])
            K.talk_prefill(plan, q.view(16 * T, -1).cuda(), keys, vc, m, gate.cuda(), out, bt, bs, blocks, T, 4, D, scale, st())
            for t in range(16 * T):
                assert relerr(out[t].view(H, D), want[t]) < TOL[dt], (window, t)


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("H,G,D,V", [(1, 1, 8, 4), (6, 2, 20, 36), (5, 5, 33, 21), (4, 2, 64, 128), (2, 1, 128, 7), (3, 1, 256, 256),
                                     (2, 2, 300, 16), (40, 8, 128, 128)])
@pytest.mark.parametrize("rot", ["none", "some", "all"])
@pytest.mark.parametrize("tiles", [False, True])
@pytest.mark.parametrize("T", [70, 300])
def test_attention_rows(K, dt, H, G, D, V, rot, tiles, T):
    """Rotation with a factor, then a norm per head of queries and keys; values as projected; rows without a cache row; keys in rows
    and in tiles."""
    from nats_llm_studio_amd.models.stack import yarn
    from nats_llm_studio_amd.models.stack_config import RotScaling
    from nats_llm_studio_amd.ops import rope_table
    d, eps, S = DT[dt], 1e-3, 304
    Dp, _ = K.head_pad(max(D, V))
    dims = {"none": 0, "some": D // 4 * 2, "all": D // 2 * 2}[rot]
    z = rnd(T, -(-((H + G) * D + G * V) // 4) * 4, seed=1).float()
    z[3] = 0
    pos = torch.arange(T) * 37 % 1000
    r = {"dims": dims, "base": 700.0, "scaling": {"factor": 5.0, "original": 100, "fast": 4.0, "slow": 0.5}}
    cs = None
    if dims:
        f, gain = yarn(700.0, dims, RotScaling(5.0, 100, 4.0, 0.5))
        cs = rope_table(1000, dims, 700.0, "cuda", f) * gain
    slot = [(5 * t) % 301 if t != 5 else -1 for t in range(T)]
    qo = torch.zeros(T, H * Dp, dtype=d, device="cuda")
    kc, vc = (torch.full((S, G * Dp), 7.0, dtype=d, device="cuda") for _ in range(2))
    zc = z.cuda()
    K.attn_rows(zc, zc[:, H * D:], zc[:, (H + G) * D:], None, None, cs, pos.int().cuda(), i32(slot), qo, kc, vc, T, H, G, D, Dp, dims,
                eps, st(), V=V, head_norm=True, key_tiles=tiles)
    if tiles:
        kc = key_rows(kc, G)
    # (columns 2 i, 2 i + 1 of a head are the pair that the plain implementation has at i, i + dims / 2)
    order = torch.cat([torch.arange(dims).view(-1, 2).T.reshape(-1), torch.arange(dims, D)])

    def plain(x, heads):
        x = x.double().view(T, heads, D)[..., order]
        return O.rms(O.rotate(x, pos, r) if dims else x, eps)
    tol = 2e-6 if dt == "f32" else 5e-3
    live = [t for t in range(T) if slot[t] >= 0]
    s = torch.tensor(slot)[live]
    qo, kc, vc = qo.cpu().view(T, H, Dp), kc.cpu().view(S, G, Dp), vc.cpu().view(S, G, Dp)
    assert relerr(qo[..., :D][..., order], plain(z[:, :H * D], H)) < tol and (qo[..., D:] == 0).all()
    assert relerr(kc[s][..., :D][..., order], plain(z[:, H * D:(H + G) * D], G)[live]) < tol
    assert torch.equal(vc[s][..., :V], z[live, (H + G) * D:(H + G) * D + G * V].view(len(live), G, V).to(d))
    assert (kc[slot[4]][..., D:] == 7).all() and (kc[5 * 5] == 7).all() and (vc[5 * 5] == 7).all()


# ---------------------------------------------------------------- embedding, norms, feed-forwards

@pytest.mark.parametrize("D", [37, 48, 1030])
def test_embedding_with_step(K, D):
    T, V = 9, 50
    tab, step = rnd(V, D, seed=1).to(torch.bfloat16), rnd(D, seed=2).float()
    ids = S.tokens(T, V, 3)
    x = torch.full((T, K.act_ld(D)), 7.0, device="cuda")
    K.embed(i32(ids), tab.cuda(), x, None, T, st(), add=step.cuda())
    assert relerr(x[:, :D], tab[ids].double() + step.double()) < 1e-6 and (x[:, D:] == 7).all()


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("D,groups", [(36, 3), (48, 16), (90, 6), (256, 2), (1024, 4), (1536, 2), (1030, 2), (2048, 8), (4096, 2),
                                      (4096, 1), (4100, 4), (8192, 4), (12288, 3), (16384, 2)])
@pytest.mark.parametrize("T", [3, 70])
def test_group_norms(K, dt, D, groups, T):
    """Both norms of a sublayer's end in one launch, parts of very different size in a row; a step vector on top; slabs; gathered
    rows."""
    d, eps, ld = DT[dt], 1e-3, K.act_ld(D)
    tol = 1e-5 if dt == "f32" else 5e-3
    w, ow, add = (rnd(D, seed=i).float() for i in (1, 2, 3))
    loud_ = torch.linspace(-2, 2, groups).exp().repeat_interleave(D // groups)
    x0, y = rnd(T, D, seed=4).float() * loud_.flip(0).float(), (rnd(2 * 128, D, seed=5) * loud_).float()
    y[1] = 0
    x, out = act(x0, ld, torch.float32), torch.zeros(T, ld, dtype=d, device="cuda")
    K.norm_add(y.cuda(), w.cuda(), x, None, T, eps, st(), out_norm=ow.cuda(), out=out, rms=True, slabs=2, slab_rows=128, groups=groups,
               add=add.cuda())
    want = x0.double() + O.norm(y[:T].double() + y[128:128 + T].double(), w.double(), eps, groups) + add.double()
    assert relerr(x[:, :D], want) < 1e-5 and (x[:, D:] == 0).all()
    after = O.norm(want, ow.double(), eps, groups)
    assert relerr(out[:, :D], after) < tol and (out[:, D:] == 0).all()
    K.row_norm(x, i32([2, 0]), ow.cuda(), out, 2, eps, st(), rms=True, groups=groups)
    assert relerr(out[:2, :D], after[[2, 0]]) < tol


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("N", [1, 7, 8, 37, 320, 2090, 12288])
@pytest.mark.parametrize("T", [1, 70])
def test_poly_norm(K, dt, N, T):
    d, eps = DT[dt], 1e-4
    z, fac = act(rnd(T, N, seed=1, scale=3.0), K.pad_to(N, 8), d), torch.tensor([0.7, -1.3, 0.4, 0.6])
    z[0] = 0
    out = torch.full((T, K.act_ld(N)), 7.0, dtype=d, device="cuda")
    K.poly_norm(z, fac.cuda(), out, N, T, eps, st())
    want = O.poly_norm(z[:, :N].double().cpu(), fac.double(), eps)
    assert relerr(out[:, :N], want) < (2e-6 if dt == "f32" else 5e-3) and (out[:, N:] == 7).all()


@pytest.mark.parametrize("E,top,groups,keep", [(12, 3, 3, 2), (16, 2, 4, 1), (5, 2, 1, 1), (1, 1, 1, 1), (6, 3, 6, 4),
                                               (64, 6, 8, 3), (200, 8, 4, 2), (512, 10, 16, 5)])
@pytest.mark.parametrize("T", [1, 3, 32, 33, 150])
def test_expert_choice(K, E, top, groups, keep, T):
    """Softmax scores over all experts, the groups' largest scores, weights as they are."""
    z = rnd(T, E, seed=E + T, scale=2.0)
    if groups > 1:
        z[0, 0] = 9.0                 # the best expert alone among weak ones: its group is kept
        z[0, 1:E // groups] = -9.0
    p = K.MoePlan(T + 9, E, top, groups, keep, 1.0, "cuda", "softmax", 1)
    p.run(z.float().cuda(), T, st())
    sel, tw = p.sel[:T * top].view(T, top).cpu(), p.topw[:T * top].view(T, top).cpu()
    for t in range(T):
        s = O.router_scores(z[t].float().double())
        want = O.choose(s, {"top": top, "groups": {"count": groups, "keep": keep}})
        assert sel[t].tolist() == want, t
        assert torch.allclose(tw[t].double(), s[want], atol=1e-6, rtol=1e-5)


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("M", [1, 20, 150, 600])
@pytest.mark.parametrize("N", [2, 50, 260])
def test_silu_gate_epilogue(K, dt, M, N):
    d, Kd = DT[dt], 72
    x, w = rnd(M, Kd, seed=5).to(d), (rnd(N, Kd, seed=10) / math.sqrt(Kd) * 3).to(d)
    y = torch.full((M, N // 2 + 5), 7.0, dtype=d, device="cuda")
    K.LinLaunch([K.Seg(K.PackedLinear(w, dt == "f32", "cuda"), act(x, K.act_ld(Kd), d), y, "siluglu", ycol=2)]).run(M, st())
    z = x.double() @ w.double().T
    assert relerr(y[:, 2:N // 2 + 2], O.silu(z[:, 0::2]) * z[:, 1::2]) < (5e-3 if dt == "bf16" else 2e-5)
    assert (y[:, :2] == 7).all() and (y[:, N // 2 + 2:] == 7).all()


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("name,i", [("uneven", 0), ("uneven", 1), ("uneven", 3), ("uneven", 4), ("ones", 0), ("ones", 1), ("wide", 0),
                                    ("wide", 2), ("split", 0)])
@pytest.mark.parametrize("T", [1, 7, 40, 230])
def test_feed_forward(K, tmp_path, dt, name, i, T):
    """A layer's second half on its own: norm, feed-forward, norm of its output."""
    from nats_llm_studio_amd.models.stack import _Step
    cfg = S.CONFIGS[name]
    W = S.make_weights(cfg)
    m = load(tmp_path, cfg, W, dt)
    b = m.step_buffers(T, 1, 16)
    x = rnd(T, cfg["width"], seed=T)
    E = cfg["layers"][i]["mlp"].get("router", {}).get("experts", 0)
    x[:, :E] = W["embed"][S.tokens(T, cfg["vocab"])][:, :E].double()          # (no close calls: see make_weights)
    layer = next(l for l, o in zip(m.layers, m.owners) if o == i)
    b.x[:T, :cfg["width"]] = x.float()
    n = cfg["norm"]
    K.row_norm(b.x, None, layer.norm_ff, b.h, T, n["eps"], st(), rms=True, groups=n["groups"])
    half = b.launches[i, "halves"]
    b.launches[i, "halves"] = [half[1]]
    keep = layer.parts, layer.after
    layer.parts, layer.after = keep[0][1:], keep[1][1:]
    layer.run(b, i, {}, None, _Step(T, 1, 16, st()), {})
    layer.parts, layer.after = keep
    p, Wd = f"l{i}.", {k: v.double() for k, v in W.items()}
    f = cfg["layers"][i]["mlp"]
    h = O.norm(x, Wd[p + "norm2"], n["eps"], n["groups"])
    y = getattr(O, O.FEED_FORWARDS[f["kind"]])(h, Wd, p + "mlp.", f, n["eps"])
    want = O.norm(y, Wd[p + "norm2b"], n["eps"], n["groups"])
    got = b.x[:T, :cfg["width"]].cpu().double() - x
    assert relerr(got, want) < (5e-5 if dt == "f32" else 4e-2)


# ---------------------------------------------------------------- whole models

@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("name", S.CONFIGS)
def test_layers_and_logits(gpu, tmp_path, dt, name):
    """The residual after every layer run, and the logits, of one prompt."""
    cfg = S.CONFIGS[name]
    W = S.make_weights(cfg)
    m = load(tmp_path, cfg, W, dt)
    toks, n = S.tokens(70, cfg["vocab"]), 70
    b = m.step_buffers(n, 1, 8, logit_rows=n)
    kc, _ = m.kv_cache(8, 16)
    pos = torch.arange(n)
    b.ids[:n], b.pos[:n], b.slot[:n] = torch.tensor(toks).int(), pos.int(), pos.int()
    b.ctx_len[:n], b.block_tables[0], b.runs[0] = (pos + 1).int(), torch.arange(8).int(), torch.tensor([0, n, 0, 0])
    taps, layers = [], []
    want = O.forward(cfg, W, toks, layers=layers)
    m.forward(b, kc, None, n, 16, logit_rows=pos.int().cuda(), n_logits=n, nruns=1, taps=taps, **m.attention_blocks(b, n))
    assert len(taps) == len(layers) == len(O.order(cfg))
    for i, (g, w) in enumerate(zip(taps, layers)):
        assert relerr(g, w) < (2e-5 if dt == "f32" else 0.06), i
    assert close(b.logits[:n].cpu(), want, dt)


def test_passes_have_their_own_caches(gpu, tmp_path):
    """The runs of a looped layer share its weights; caches are each run's own."""
    cfg = S.CONFIGS["uneven"]
    m = load(tmp_path, cfg, S.make_weights(cfg), "bf16")
    assert m.owners == [0, 1, 2, 3, 1, 2, 3, 1, 2, 3, 4] and m.layers[1] is m.layers[4] is m.layers[7]
    kc = m.kv_cache(4, 16)[0]
    assert set(kc) == set(range(11)) and len({c.data_ptr() for c in kc.values()}) == 11 and not m.state_pool(2)
    assert m.kv_token_bytes == sum(c[0][0].shape[-1] * 4 for c in kc.values()) and not m.recurrent


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("name", S.CONFIGS)
def test_feed_schedules(gpu, tmp_path, dt, name):
    """One sequence whole, token by token, and in portions of several sizes; three unequal ones mixed, in reused pages: always the
    plain implementation's logits."""
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
    assert eng.alloc.n_free == eng.num_blocks
    assert eng.counters["graph_replays"] > 20


@pytest.mark.parametrize("dt", DT)
def test_batch_independence(gpu, tmp_path, dt):
    """A prompt's logits next to others, and in other pages, are those it has alone, beyond rounding."""
    cfg = S.CONFIGS["uneven"]
    m = load(tmp_path, cfg, S.make_weights(cfg), dt)
    b = m.step_buffers(512, 4, 16, logit_rows=512)
    kc, _ = m.kv_cache(40, 16)
    ps = [S.tokens(n, cfg["vocab"], n) for n in (3, 81, 130, 2)]
    blk = [[0], [3, 1, 9, 30, 31, 5], list(range(10, 19)), [39]]
    alone = [run_rows(m, b, kc, None, [(0, list(range(20, 30)), 0, p)])[0] for p in ps]
    for order in ((0, 1, 2, 3), (2, 3, 1, 0)):
        got = run_rows(m, b, kc, None, [(3 - i, blk[i], 0, ps[i]) for i in order])
        for i, g in zip(order, got):
            assert close(g, alone[i].double(), dt)


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("far,seen", [(0, (0, 0)), (209, (0, 0)), (210, (1, 0)), (248, (1, 0)), (249, (1, 1)), (358, (1, 1)),
                                      (360, (0, 1))])
def test_single_keys(gpu, tmp_path, dt, far, seen):
    """Two queries at places 359 and 398 with a window of 150: one key among hundreds, just inside or outside of what they see. Its
    exchange shows where it is seen and nowhere else, in a prompt and when decoding."""
    cfg = S.config([S.layer(S.attention(4, 2, 16, 16, 1.5, 150, dims=0))], width=64, vocab=99, groups=1)
    W = S.make_weights(cfg)
    # token 97 has a direction e, token 98 a direction f that no other token has, and a query sees f as a key sees e
    e, f = torch.linalg.qr(torch.randn(64, 2, generator=torch.Generator().manual_seed(8)))[0].T
    emb = W["embed"].float()
    emb -= (emb @ e)[:, None] * e + (emb @ f)[:, None] * f
    emb[97], emb[98] = 0.2 * emb[97] + 5 * e, 0.2 * emb[98] + 5 * f
    W["embed"], W["l0.norm1"] = emb.to(torch.bfloat16), torch.ones(64, dtype=torch.bfloat16)
    k = W["l0.mix.k"].float()
    kq = (k + torch.outer(k @ (e - f), f)).view(2, 1, 16, 64).expand(2, 2, 16, 64)
    W["l0.mix.q"] = kq.reshape(64, 64).to(torch.bfloat16)
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
    c = S.config([S.layer(S.attention(), S.dense()), S.layer(S.attention(4, 4, 16, 32, 0.4, 9, 8), S.moe())], loop=(0, 2, 2))
    W = S.make_weights(c)
    reqs = [(S.tokens(6 + 11 * i, c["vocab"], 20 + i), 24 - 2 * i) for i in range(6)]
    return c, W, reqs, [greedy(c, W, p, n) for p, n in reqs]


@pytest.mark.parametrize("blocks,graphs", [(64, True), (64, False), (7, True)])
def test_generation(gpu, tmp_path, blocks, graphs, expected):
    """Greedy generation of six requests over three decode rows, with and without graphs, and over a pool so small that
    sequences are preempted and prefilled again; the same prompt again finds its pages cached."""
    from nats_llm_studio_amd.engine.engine import GenRequest
    from nats_llm_studio_amd.engine.sampling import SamplingParams
    cfg, W, reqs, want = expected
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
    assert blocks == 64 or eng.counters["preemptions"] > 0
    assert not graphs or eng.counters["graph_replays"] > 0
    if blocks == 64:
        hits = eng.alloc.hits
        r = eng.generate(reqs[5][0], SamplingParams(max_tokens=reqs[5][1], ignore_eos=True))
        assert r.token_ids == want[5] and eng.alloc.hits > hits


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
    S.write_model(str(tmp_path / "pub" / "pimo"), cfg, W)
    reg = Registry(str(tmp_path))
    reg.scan()
    be = EngineBackend(WorkerConfig(models_dir=str(tmp_path), device="cuda:0", max_batch=4, max_ctx=256, dtype="float32",
                                    max_prefill_tokens=256))
    got, ev = [], threading.Event()

    def done(status, body, *a):
        got.append((status, body))
        ev.set()
    be.chat("pimo", reg.resolve("pimo"), {"messages": [{"role": "user", "content": "5 17 3 99"}], "max_tokens": 6,
                                          "ignore_eos": True}, done)
    assert ev.wait(100)
    status, body = got[0]
    assert status == 200, body
    assert body["model_info"]["arch"] == "Pimodra"
    assert [int(t) for t in body["choices"][0]["message"]["content"].split()] == greedy(cfg, W, [5, 17, 3, 99], 6)
    assert be.unload("pimo")
