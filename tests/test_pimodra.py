"""Pimodra on the CPU: configuration, order of the looped layers, and the plain implementation against itself (cut sequences,
hand-computed values, planted mistakes). The kernels are in test_pimodra_gpu.py."""
import json
import math

import pytest
import torch

import pimodra_models as S
import pimodra_oracle as O
from nats_llm_studio_amd.models.registry import checkpoint_kind, stack_arch, supported_architectures
from nats_llm_studio_amd.models.stack import yarn
from nats_llm_studio_amd.models.stack_config import RotScaling, StackConfig


def shapes(W):
    return lambda n: tuple(W[n].shape) if n in W else None


@pytest.mark.parametrize("name", S.CONFIGS)
def test_config(name):
    cfg = S.CONFIGS[name]
    W = S.make_weights(cfg)
    c = StackConfig.from_json(cfg, shapes(W))
    assert (c.d_model, c.vocab, c.eps, c.norm_groups) == (cfg["width"], cfg["vocab"], cfg["norm"]["eps"], cfg["norm"]["groups"])
    assert (c.embed_scale, c.softcap, c.recurrent, c.n_layer) == (1.0, 0.0, False, len(cfg["layers"])) and c.order == O.order(cfg)
    for L, l in zip(cfg["layers"], c.layers):
        m, j = l.mixer, L["mixer"]
        assert m.kind == "attention" and all(getattr(m, k) == j[k] for k in ("heads", "kv_heads", "dim", "vdim", "scale"))
        assert (m.window, m.keep_first) == (j["mask"]["size"], 0)
        rot = j.get("rot", {"dims": 0, "base": 1.0})
        assert (m.rot_dims, m.rot_base) == (rot["dims"], rot["base"])
        assert m.rot_scaling == (RotScaling(**rot["scaling"]) if "scaling" in rot else None)
        f = L["mlp"]
        if f is None:
            assert l.mlp is None
        elif f["kind"] == "dense":
            assert l.mlp.kind == "dense" and l.mlp.ff == f["ff"]
        else:
            g = f["router"].get("groups", {"count": 1, "keep": 1})
            assert (l.mlp.experts, l.mlp.top, l.mlp.ff, l.mlp.groups, l.mlp.keep, l.mlp.scale, l.mlp.shared_ff) == (
                f["router"]["experts"], f["router"]["top"], f["expert"]["ff"], g["count"], g["keep"], 1.0, 0)
    # sizes that the config leaves out come from the tensors
    lean = json.loads(json.dumps(cfg))
    for k in ("width", "vocab"):
        lean.pop(k)
    for L in lean["layers"]:
        for k in ("heads", "kv_heads", "dim", "vdim"):
            L["mixer"].pop(k)
        if L["mlp"] and L["mlp"]["kind"] == "dense":
            L["mlp"].pop("ff")
        elif L["mlp"]:
            L["mlp"].pop("expert")
            L["mlp"]["router"].pop("experts")
    for L in lean["layers"]:             # (a key size has no tensor of its own: it follows from the heads)
        assert "dim" not in L["mixer"]
    assert StackConfig.from_json(lean, shapes(W)) == c


def test_config_refusals():
    def bad(edit, exc=ValueError, name="uneven"):
        c = json.loads(json.dumps(S.CONFIGS[name]))
        edit(c)
        with pytest.raises(exc):
            StackConfig.from_json(c)
    bad(lambda c: c["layers"][0].update(type="lightning"), NotImplementedError)       # not a mixer of this design
    bad(lambda c: c["layers"][0]["mixer"].update(kv_heads=4))                         # 6 heads over 4
    bad(lambda c: c["layers"][0]["mixer"]["mask"].update(size=0))
    bad(lambda c: c["layers"][0]["mixer"]["mask"].update(keep_first=3), NotImplementedError)
    bad(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=22))                     # heads of 20
    bad(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7))
    bad(lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=0))
    bad(lambda c: c["layers"][1]["mlp"]["router"].update(top=7))                      # 3 groups of 2 kept
    bad(lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=4))
    bad(lambda c: c["norm"].update(groups=3))                                         # 136 columns
    bad(lambda c: c["loop"].update(stop=9))
    bad(lambda c: c["loop"].update(times=0))


def test_registry(tmp_path):
    cfg = S.CONFIGS["ones"]
    d = S.write_model(str(tmp_path / "pub" / "Tiny-Pimodra"), cfg, S.make_weights(cfg))
    assert checkpoint_kind(d) == "stack" and stack_arch(d) == "Pimodra" and "Pimodra" in supported_architectures()
    from nats_llm_studio_amd.service.registry import Registry
    reg = Registry(str(tmp_path))
    (e,) = reg.scan()
    assert e.id == "tiny-pimodra" and e.arch == "Pimodra" and e.quantization == "BF16" and e.path == d


@pytest.mark.parametrize("dims,base,s", [(12, 900.0, S.scaling()), (64, 1e4, S.scaling(8.0, 2048, 32.0, 1.0)), (2, 5.0, S.scaling()),
                                         (8, 50.0, S.scaling(2.0, 7, 1.0, 1.0)), (16, 1e6, S.scaling(1.0, 64, 2.0, 1.0)),
                                         (10, 3.0, S.scaling(4.0, 1e6, 100.0, 50.0))])
def test_rotation_scaling(dims, base, s):
    """Frequencies and gain of the product against the plain ones, ramps cut at both ends and of no length among them."""
    want, gain = O.frequencies({"dims": dims, "base": base, "scaling": s})
    div, g = yarn(base, dims, RotScaling(**s))
    got = [base ** (-2.0 * i / dims) / d for i, d in enumerate(div)]
    assert g == pytest.approx(gain) and got == pytest.approx(want, rel=1e-12)


def test_launch_plans():
    """Kernels and scratch of the attention with mixed heads."""
    from nats_llm_studio_amd.ops import stack as K
    p = K.TalkPlan(32, 8, 128, 1024, 8192, False, "cpu")
    assert p.mfma and p.prefill and p.ks == 1056 and p.rows(4096) * p.ks * p.hs * 4 <= K.TALK_SCRATCH
    for T in (1, 2, 7, 64, 256, 1000):
        ns1, ns, waves = p.splits(T)
        assert 1 <= ns1 <= 64 and 1 <= ns <= 64 and waves in (1, 4)
        sc, ss, po, cnt = p.scratch(T)
        assert sc >= min(T, p.rows(T)) * p.ks * p.hs and ss >= T * ns1 * p.hs * 2 and cnt >= T * p.groups
        assert ns == 1 or po >= T * ns * 32 * 128
    assert not K.TalkPlan(40, 8, 128, 0, 512, False, "cpu").prefill and K.TalkPlan(40, 8, 128, 0, 512, False, "cpu").mfma
    assert not K.TalkPlan(130, 10, 32, 0, 512, False, "cpu").mfma and not K.TalkPlan(4, 2, 32, 0, 512, True, "cpu").mfma
    assert not K.TalkPlan(4, 2, 32, 0, 512, False, "cpu", scale=-1.0).prefill
    m = K.TalkPlan(5, 5, 32, 9, 512, False, "cpu").matrix(torch.ones(5, 5, dtype=torch.bfloat16))
    assert m.shape == (32, 32) and float(m.sum()) == 25.0 and float(m[:5, :5].sum()) == 25.0


# ---- the plain implementation against itself

@pytest.mark.parametrize("i", [0, 1, 3])
def test_oracle_cut_sequences(i):
    """A mixer fed in pieces, with carried keys and values, equals one pass."""
    cfg = S.CONFIGS["uneven"]
    W = {k: v.double() for k, v in S.make_weights(cfg).items()}
    L, eps = cfg["layers"][i], cfg["norm"]["eps"]
    h = torch.randn(83, cfg["width"], generator=torch.Generator().manual_seed(3), dtype=torch.float64)
    pos = torch.arange(83)
    whole, _ = O.attention_mixer(h, W, f"l{i}.mix.", L["mixer"], pos, eps)
    before, out = None, []
    for a, b in ((0, 1), (1, 3), (3, 16), (16, 83)):
        y, before = O.attention_mixer(h[a:b], W, f"l{i}.mix.", L["mixer"], pos[a:b], eps, before)
        out.append(y)
    assert torch.allclose(torch.cat(out), whole, atol=1e-10)


def test_oracle_known_values():
    """Hand-computed cases."""
    x = torch.tensor([[3.0, 4.0, 0.0, 2.0]]).double()
    w = torch.tensor([1.0, 2.0, 1.0, 0.5]).double()
    # parts (3, 4) and (0, 2): mean squares 12.5 and 2
    want = torch.tensor([[3 / 13 ** 0.5, 8 / 13 ** 0.5, 0.0, 1 / 2.5 ** 0.5]]).double()
    assert torch.allclose(O.norm(x, w, 0.5, 2), want)
    assert torch.allclose(O.norm(x, w, 0.5, 1), x * w / (29 / 4 + 0.5) ** 0.5)
    i, j = torch.tensor([9])[:, None], torch.arange(12)[None]
    assert O.visible(i, j, {"size": 3})[0].nonzero().flatten().tolist() == [7, 8, 9]
    assert O.visible(i, j, None)[0].sum() == 10
    # two heads over two keys: weights (1/5, 4/5) and (1/2, 1/2); the second head's become 2 w0 - w1, the first's w1
    q = torch.tensor([[[1.0], [0.0]]]).double()
    k = torch.tensor([[[0.0], [0.0]], [[math.log(4.0)], [0.0]]]).double()
    v = torch.tensor([[[1.0], [10.0]], [[3.0], [20.0]]]).double()
    talk = torch.tensor([[0.0, 1.0], [2.0, -1.0]]).double()
    o = O.attend(q, k, v, torch.tensor([1]), 1.0, None, talk).flatten().tolist()
    assert o == pytest.approx([0.5 * 1 + 0.5 * 3, (0.4 - 0.5) * 10 + (1.6 - 0.5) * 20])
    # a head of four, two of them rotated by 90 degrees at position 1: (u, v) -> (-v, u), the other two stay
    f = O.frequencies({"dims": 2, "base": 7.0})
    assert f == ([1.0], 1.0)
    r = O.rotate(torch.tensor([[[1.0, 2.0, 5.0, 6.0]]]).double(), torch.tensor([math.pi / 2]).double(), {"dims": 2, "base": 7.0})
    assert torch.allclose(r, torch.tensor([[[-2.0, 1.0, 5.0, 6.0]]]).double())
    # long wavelengths by the factor, short ones as they are
    f, g = O.frequencies({"dims": 8, "base": 16.0, "scaling": {"factor": 10.0, "original": 2 * math.pi * 8, "fast": 8.0, "slow": 1.0}})
    # turns: 8 -> pair 0, 1 -> pair 3
    assert f == pytest.approx([1.0, 0.5 * (1 - 0.9 / 3), 0.25 * (1 - 0.9 * 2 / 3), 0.0125]) and g == pytest.approx(1 + 0.1 * math.log(10))
    z = torch.tensor([[1.0, -1.0, 1.0, -1.0]]).double()
    assert torch.allclose(O.poly_norm(z, torch.tensor([1.0, 2.0, 4.0, 8.0]).double(), 0.0), torch.tensor([[15.0, 5.0, 15.0, 5.0]]).double())
    s = O.router_scores(torch.log(torch.tensor([1.0, 2.0, 3.0, 4.0])).double())
    assert s.tolist() == pytest.approx([0.1, 0.2, 0.3, 0.4])
    assert O.choose(s, {"top": 2}) == [3, 2]
    # groups (.4, .3), (.05, .25): the second is left out
    assert O.choose(torch.tensor([0.4, 0.05, 0.3, 0.25]), {"top": 2, "groups": {"count": 2, "keep": 1}}) == [0, 1]


def _window(n):
    return lambda i, j, mask, f=O.visible: f(i, j, mask and dict(size=mask["size"] + n))


def _interleaved(x, positions, rot):
    f, gain = O.frequencies(rot)
    out = x.clone()
    for i, v in enumerate(f):
        a = positions.to(x.dtype) * v
        c, s = (torch.cos(a) * gain)[:, None], (torch.sin(a) * gain)[:, None]
        out[:, :, 2 * i] = x[:, :, 2 * i] * c - x[:, :, 2 * i + 1] * s
        out[:, :, 2 * i + 1] = x[:, :, 2 * i + 1] * c + x[:, :, 2 * i] * s
    return out


def _mix_scores(q, k, v, positions, scale, mask, talk):
    H, G = q.shape[1], k.shape[1]
    see = O.visible(positions[:, None], torch.arange(k.shape[0])[None, :], mask)
    s = O.mix_heads(torch.stack([q[:, h] @ k[:, h // (H // G)].T * scale for h in range(H)]), talk).masked_fill(~see, -math.inf)
    w = torch.softmax(s, -1)
    return torch.stack([w[h] @ v[:, h // (H // G)] for h in range(H)], 1)


def _layer(pre=True, post=True, order=False):
    def f(x, W, p, L, positions, nrm, before=None):
        eps, groups = nrm["eps"], nrm["groups"]
        n = lambda v, name: O.norm(v, W[p + name], eps, groups)      # noqa: E731
        y, after = O.attention_mixer(n(x, "norm1") if pre else x, W, p + "mix.", L["mixer"], positions, eps, before)
        x0, x = x, x + (n(y, "norm1b") if post else y)
        if L.get("mlp"):
            y = getattr(O, O.FEED_FORWARDS[L["mlp"]["kind"]])(n(x0 if order else x, "norm2"), W, p + "mlp.", L["mlp"], eps)
            x = x + (n(y, "norm2b") if post else y)
        return x, after
    return f


def _no_group(s, router, f=O.choose):
    return f(s, dict(router, groups=None))


MISTAKES = {
    "the window is one short": ("visible", _window(-1)),
    "the window is one long": ("visible", _window(1)),
    "the heads are not mixed": ("mix_heads", lambda w, talk: w),
    "the matrix is transposed": ("mix_heads", lambda w, talk, f=O.mix_heads: f(w, talk.T)),
    "the scores are mixed, not the weights": ("attend", _mix_scores),
    "there is no output gate": ("output_gate", lambda o, h, wg: o),
    "pairs of neighbours are rotated": ("rotate", _interleaved),
    "nothing is rotated": ("rotate", lambda x, positions, rot: x),
    "the rotation is not scaled": ("frequencies", lambda rot, f=O.frequencies: f(dict(rot, scaling=None))),
    "the rotation has no gain": ("frequencies", lambda rot, f=O.frequencies: (f(rot)[0], 1.0)),
    "the norms have one group": ("norm", lambda x, w, eps, groups, f=O.norm: f(x, w, eps, 1)),
    "there is no norm ahead": ("layer", _layer(pre=False)),
    "there is no norm behind": ("layer", _layer(post=False)),
    "the feed-forward reads the old residual": ("layer", _layer(order=True)),
    "the square is left out": ("poly_norm", lambda z, a, eps, f=O.poly_norm: f(z, a * torch.tensor([1, 0, 1, 1]), eps)),
    "the cube is left out": ("poly_norm", lambda z, a, eps, f=O.poly_norm: f(z, a * torch.tensor([1, 1, 0, 1]), eps)),
    "the constant is left out": ("poly_norm", lambda z, a, eps, f=O.poly_norm: f(z, a * torch.tensor([1, 1, 1, 0]), eps)),
    "the powers are of the normed values": ("poly_norm", lambda z, a, eps, f=O.poly_norm: (
        a[0] * O.rms(z, eps) + a[1] * O.rms(z, eps) ** 2 + a[2] * O.rms(z, eps) ** 3 + a[3])),
    "the groups' scores are sums": ("group_score", lambda s: s.sum()),
    "the groups are ignored": ("choose", _no_group),
    "every pass has the first one's step": ("enter_pass", lambda x, W, t, f=O.enter_pass: f(x, W, 0)),
    "only the first pass is entered": ("enter_pass", lambda x, W, t, f=O.enter_pass: f(x, W, t) if t == 0 else x),
}


@pytest.mark.parametrize("mistake", MISTAKES)
def test_weights_show_mistakes(mistake, monkeypatch):
    """The tests' weights make each mistake visible well above what bf16 rounding does (test_pimodra_gpu.WHOLE)."""
    cfg = S.CONFIGS["uneven"]
    W, toks = S.make_weights(cfg), S.tokens(72, cfg["vocab"], 5)
    good = O.forward(cfg, W, toks)
    monkeypatch.setattr(O, *MISTAKES[mistake])
    e = S.error(O.forward(cfg, W, toks), good)
    print(mistake, round(e, 3))
    assert e > 0.12


def test_bench_option_parses():
    import bench
    assert bench.parse(["--stack", "all", "--stack-design", "pimodra"]).stack_design == "pimodra"
    from nats_llm_studio_amd import bench_stack
    for size in bench_stack.SIZES["pimodra"].values():
        c = StackConfig.from_json(bench_stack.CONFIGS["pimodra"](size))
        assert [L.mlp.kind for L in c.layers] == ["dense", "moe", "moe"] and len(c.order) == 4
