"""Bibapel on the CPU: configuration, order of the looped layers, and the plain implementation against itself (cut sequences,
hand-computed values, planted mistakes). The kernels are in test_bibapel_gpu.py."""
import json
import math

import pytest
import torch

import bibapel_models as S
import bibapel_oracle as O
from nats_llm_studio_amd.models.registry import checkpoint_kind, stack_arch, supported_architectures
from nats_llm_studio_amd.models.stack_config import StackConfig


def shapes(W):
    return lambda n: tuple(W[n].shape) if n in W else None


@pytest.mark.parametrize("name", S.CONFIGS)
def test_config(name):
    cfg = S.CONFIGS[name]
    W = S.make_weights(cfg)
    c = StackConfig.from_json(cfg, shapes(W))
    b = cfg["embedding"]["bigram"]
    assert (c.d_model, c.vocab, c.eps, c.n_layer) == (cfg["width"], cfg["vocab"], cfg["norm"]["eps"], len(cfg["layers"]))
    assert (c.embed_scale, c.softcap, c.n_expert, c.recurrent) == (cfg["embedding"]["scale"], 0.0, 0, True)
    assert (c.bigram.buckets, c.bigram.mul_prev, c.bigram.mul_cur) == (b["buckets"], b["mul_prev"], b["mul_cur"])
    assert c.max_positions == cfg["max_positions"] and c.ctx <= c.max_positions
    assert c.order == O.order(cfg)
    for L, l in zip(cfg["layers"], c.layers):
        m = l.mixer
        assert m.kind == L["type"] and all(getattr(m, k) == v for k, v in L["mixer"].items() if k != "mask")
        if m.kind == "attention":
            k = L["mixer"].get("mask", {"size": 0, "keep_first": 0})
            assert (m.window, m.keep_first, m.rot_dims) == (k["size"], k["keep_first"], 0)
        assert ((l.mlp.ff, l.mlp.limit) if l.mlp else None) == ((L["mlp"]["ff"], L["mlp"]["limit"]) if L["mlp"] else None)
    # sizes that the config leaves out come from the tensors
    lean = json.loads(json.dumps(cfg))
    for k in ("width", "vocab", "max_positions"):
        lean.pop(k)
    lean["embedding"]["bigram"].pop("buckets")
    for L in lean["layers"]:
        drop = {"channel_delta": ("heads", "kv_heads", "dim", "vdim", "conv"), "attention": ("kv_heads", "dim", "vdim"),
                "lightning": ("heads", "dim", "vdim")}[L["type"]]
        for k in drop:
            L["mixer"].pop(k)
        if L["mlp"]:
            L["mlp"].pop("ff")
    assert StackConfig.from_json(lean, shapes(W)) == c


def test_config_refusals():
    def bad(edit, exc=ValueError, name="uneven"):
        c = json.loads(json.dumps(S.CONFIGS[name]))
        edit(c)
        with pytest.raises(exc):
            StackConfig.from_json(c)
    bad(lambda c: c["layers"][0].update(type="gla"), NotImplementedError)             # not a mixer of this design
    bad(lambda c: c["layers"][1]["mlp"].update(kind="moe"), NotImplementedError)
    bad(lambda c: c["layers"][2]["mixer"].update(kv_heads=4))                         # 6 heads over 4
    bad(lambda c: c["layers"][1]["mixer"].update(kv_heads=3))
    bad(lambda c: c["layers"][2]["mixer"]["mask"].update(size=0))
    bad(lambda c: c["layers"][0]["mixer"].update(decay=[0.5, 0.5]))                   # 3 heads
    bad(lambda c: c["layers"][0]["mixer"]["decay"].__setitem__(1, 1.5))
    bad(lambda c: c["loop"].update(stop=9))
    bad(lambda c: c["loop"].update(times=0))
    bad(lambda c: c["loop"].update(start=4))
    bad(lambda c: c["embedding"]["bigram"].update(buckets=0))


def test_order_of_runs():
    """Each pass has its own runs (and with them its own caches and states); its number is told ahead of its first layer."""
    c = StackConfig.from_json(S.CONFIGS["uneven"])
    assert c.order == [(0, None)] + [(1, 0), (2, None), (3, None), (1, 1), (2, None), (3, None), (1, 2), (2, None), (3, None)] + [
        (4, None), (5, None)]
    c = StackConfig.from_json(S.CONFIGS["big heads"])
    assert c.order == [(0, 0), (0, 1), (1, None), (2, None)]
    c = StackConfig.from_json(S.CONFIGS["odd"])
    assert c.order == [(i, None) for i in range(4)]


def test_registry(tmp_path):
    cfg = S.CONFIGS["ones"]
    d = S.write_model(str(tmp_path / "pub" / "Tiny-Bibapel"), cfg, S.make_weights(cfg))
    assert checkpoint_kind(d) == "stack" and stack_arch(d) == "Bibapel" and "Bibapel" in supported_architectures()
    from nats_llm_studio_amd.service.registry import Registry
    reg = Registry(str(tmp_path))
    (e,) = reg.scan()
    assert e.id == "tiny-bibapel" and e.arch == "Bibapel" and e.quantization == "BF16" and e.path == d


def test_launch_shapes():
    """Segments of the delta rule: at least 128 tokens each, none for decoding or for many runs."""
    from nats_llm_studio_amd.ops import stack as K
    for T, n, H, V in ((1, 1, 4, 64), (7, 7, 2, 20), (260, 3, 2, 64), (4096, 1, 32, 128), (4096, 4, 4, 512)):
        nseg, nt = K.delta_shape(T, n, H, 64, V)
        assert 1 <= nseg <= 16 and (nseg == 1 or (T - n + 1) // nseg >= 128) and nt == (1 if V <= 64 else 2)
    assert K.delta_shape(4096, 1, 4, 64, 64)[0] == 16 and K.delta_shape(4096, 8, 32, 64, 128)[0] == 1


# ---- the plain implementation against itself

@pytest.mark.parametrize("i", [0, 1, 2, 5])
def test_oracle_cut_sequences(i):
    """A mixer fed in pieces, with carried keys, states and convolution inputs, equals one pass."""
    cfg = S.CONFIGS["uneven"]
    W = {k: v.double() for k, v in S.make_weights(cfg).items()}
    L, eps = cfg["layers"][i], cfg["norm"]["eps"]
    f = getattr(O, O.MIXERS[L["type"]])
    h = torch.randn(83, cfg["width"], generator=torch.Generator().manual_seed(3), dtype=torch.float64)
    pos = torch.arange(83)
    whole, _ = f(h, W, f"l{i}.mix.", L["mixer"], pos, eps)
    before, out = None, []
    for a, b in ((0, 1), (1, 3), (3, 16), (16, 83)):
        y, before = f(h[a:b], W, f"l{i}.mix.", L["mixer"], pos[a:b], eps, before)
        out.append(y)
    assert torch.allclose(torch.cat(out), whole, atol=1e-10)


def test_oracle_embedding():
    """The pair's row, the first token's row, the position's vector; a sequence embedded in two pieces."""
    cfg = {"embedding": {"scale": 0.5, "bigram": {"buckets": 7, "mul_prev": 3, "mul_cur": 2}}}
    W = {"embed": torch.tensor([[2.0], [4.0], [6.0], [8.0], [10.0], [12.0]]), "bigram": 100.0 * torch.arange(8.0)[:, None],
         "pos": 0.125 * torch.arange(9.0)[:, None]}
    # rows: the last one, (5 * 3 + 1 * 2) % 7 = 3, (1 * 3 + 3 * 2) % 7 = 2
    assert O.embed(cfg, W, [5, 1, 3]).flatten().tolist() == [706.0, 302.125, 204.25]
    assert O.embed(cfg, W, [3], prev=1, first=2).flatten().tolist() == [204.25]


def test_oracle_known_values():
    """Hand-computed cases."""
    x = torch.tensor([[3.0, 4.0]])
    assert torch.allclose(O.norm(x, torch.tensor([0.5, 2.0]), 0.5), x / 13.0 ** 0.5 * torch.tensor([0.5, 2.0]))
    assert torch.allclose(O.unit(x), x / 5.0, atol=1e-6)
    # the window's edge and the kept tokens
    i, j = torch.tensor([9])[:, None], torch.arange(12)[None]
    assert O.visible(i, j, {"size": 3, "keep_first": 2})[0].nonzero().flatten().tolist() == [0, 1, 7, 8, 9]
    assert O.visible(i, j, None)[0].sum() == 10
    # a query with equal scores of log 2 on two keys: weights 2 / 5 each
    q, k = torch.ones(1, 1, 1).double(), torch.full((2, 1, 1), math.log(2.0)).double()
    v = torch.tensor([[[1.0]], [[4.0]]]).double()
    assert torch.allclose(O.attend(q, k, v, torch.tensor([1]), 1.0, None), torch.tensor(2.0).double())
    # a group's heads share their key head: 4 query heads, 2 key heads
    q, k = torch.zeros(1, 4, 1).double(), torch.zeros(1, 2, 1).double()
    v = torch.tensor([[[1.0], [2.0]]]).double()
    assert O.attend(q, k, v, torch.tensor([0]), 1.0, None).flatten().tolist() == [0.5, 0.5, 1.0, 1.0]
    one = lambda *v: torch.tensor(v, dtype=torch.float64).view(len(v), 1, 1)      # noqa: E731
    o, s = O.lightning_scan(one(1.0, 2.0), one(2.0, 3.0), one(5.0, 7.0), torch.tensor([0.5]).double())
    assert o.flatten().tolist() == [10.0, 52.0] and float(s) == 26.0
    # delta rule: S = 0.5 * 4 = 2, answer 2 * 2 = 4, u = 0.25 * (8 - 4) = 1, S = 2 + 2 = 4, read 3 * 4
    o, s = O.delta_scan(one(3.0), one(2.0), one(8.0), one(0.5), torch.tensor([[0.25]]).double(), one(4.0))
    assert float(o) == 12.0 and float(s) == 4.0
    y, tail = O.causal_conv(torch.tensor([[1.0], [2.0], [3.0]]), torch.tensor([[10.0, 1.0]]))
    assert y.flatten().tolist() == [1.0, 12.0, 23.0] and tail.flatten().tolist() == [3.0]
    # clamped feed-forward: gate 9 -> 2, up 9 -> 2; gate -9 stays, up -9 -> -2
    W = {"gate": torch.tensor([[9.0]]), "up": torch.tensor([[9.0]]), "down": torch.tensor([[1.0]])}
    sg = lambda z: 1 / (1 + math.exp(-z))      # noqa: E731
    y = O.dense_ff(torch.tensor([[1.0], [-1.0]]), W, "", 2.0).flatten().tolist()
    assert y == pytest.approx([2 * sg(3.404) * 3, -9 * sg(-15.318) * -1], rel=1e-4)


def _conv_reversed(x, w, before=None, f=O.causal_conv):
    return f(x, w.flip(1), before)


def _delta_order(decay_last=False, read_first=False, no_correction=False):
    def f(q, k, v, g, beta, state=None):
        S, out = torch.zeros(q.shape[1], q.shape[2], v.shape[2]).double(), []
        for t in range(q.shape[0]):
            if not decay_last:
                S = g[t][:, :, None] * S
            if read_first:
                out.append((S * q[t][:, :, None]).sum(1))
            a = 0.0 if no_correction else (S * k[t][:, :, None]).sum(1)
            S = S + k[t][:, :, None] * (beta[t][:, None] * (v[t] - a))[:, None, :]
            if decay_last:
                S = g[t][:, :, None] * S
            if not read_first:
                out.append((S * q[t][:, :, None]).sum(1))
        return torch.stack(out), S
    return f


def _delta_lost(q, k, v, g, beta, state=None, f=O.delta_scan):
    return torch.cat([f(*(t[s] for t in (q, k, v, g, beta)))[0] for s in (slice(20), slice(20, None))]), None


def _lightning_lost(q, k, v, decay, state=None, f=O.lightning_scan):
    return torch.cat([f(q[s], k[s], v[s], decay)[0] for s in (slice(20), slice(20, None))]), None


def _window(size=0, keep=0):
    return lambda i, j, mask, f=O.visible: f(i, j, mask and dict(size=mask["size"] + size, keep_first=max(0, mask["keep_first"] + keep)))


def _bigram(first=False, swap=False):
    def f(prev, cur, b, g=O.bigram_row):
        if prev is None:
            return g(0, cur, b) if first else g(None, cur, b)
        return g(cur, prev, b) if swap else g(prev, cur, b)
    return f


def _ff(low=False, one=True, plain=False):
    def f(h, W, p, limit):
        g = torch.clamp(h @ W[p + "gate"].T, max=limit, min=-limit if low else None)
        u = torch.clamp(h @ W[p + "up"].T, min=-limit, max=limit)
        return (g * O.sigmoid(g if plain else 1.702 * g) * (u + (1.0 if one else 0.0))) @ W[p + "down"].T
    return f


def _one_norm(x, W, p, L, positions, eps, before=None, f=O.layer):
    return f(x, dict(W, **{p + "norm2": W[p + "norm1"]}) if L.get("mlp") else W, p, L, positions, eps, before)


def _in_series(x, W, p, L, positions, eps, before=None):
    y, after = getattr(O, O.MIXERS[L["type"]])(O.norm(x, W[p + "norm1"], eps), W, p + "mix.", L["mixer"], positions, eps, before)
    x = x + y
    if L.get("mlp"):
        x = x + O.dense_ff(O.norm(x, W[p + "norm2"], eps), W, p + "mlp.", L["mlp"]["limit"])
    return x, after


def _per_head_norm(h, W, p, m, positions, eps, before=None):
    H, V = m["heads"], m["vdim"]
    q, k, v = (O.silu(h @ W[p + n].T).reshape(h.shape[0], H, -1) for n in "qkv")
    o, S = O.lightning_scan(q, k, v, torch.tensor(m["decay"], dtype=h.dtype))
    o = O.rms(o, eps).reshape(h.shape[0], H * V) * W[p + "norm"] * O.sigmoid(h @ W[p + "g"].T)
    return o @ W[p + "o"].T, S


MISTAKES = {
    "the window is one short": ("visible", _window(size=-1)),
    "the window is one long": ("visible", _window(size=1)),
    "one kept token is missed": ("visible", _window(keep=-1)),
    "one more token is kept": ("visible", _window(keep=1)),
    "the sink is left out": ("sink_weights", lambda e, one: e / e.sum(-1, keepdim=True)),
    "there is no decay": ("delta_decay", lambda *a, f=O.delta_decay: torch.ones_like(f(*a))),
    "the decay comes after the write": ("delta_scan", _delta_order(decay_last=True)),
    "the state is read before the write": ("delta_scan", _delta_order(read_first=True)),
    "nothing is corrected": ("delta_scan", _delta_order(no_correction=True)),
    "the delta state is lost at token 20": ("delta_scan", _delta_lost),
    "the lightning state is lost at token 20": ("lightning_scan", _lightning_lost),
    "the taps are reversed": ("causal_conv", _conv_reversed),
    "the convolution starts anew at token 20": ("causal_conv", lambda x, w, b=None, f=O.causal_conv: (
        torch.cat([f(x[:20], w)[0], f(x[20:], w)[0]]), f(x, w)[1])),
    "keys and queries are no unit vectors": ("unit", lambda x: x),
    "the outputs are normed per head": ("lightning_mixer", _per_head_norm),
    "the first token has a pair": ("bigram_row", _bigram(first=True)),
    "the pair is swapped": ("bigram_row", _bigram(swap=True)),
    "positions start at one": ("embed", lambda cfg, W, toks, prev=None, first=0, f=O.embed: f(cfg, W, toks, prev, 1)),
    "the gate is clamped below": ("dense_ff", _ff(low=True)),
    "up has no one added": ("dense_ff", _ff(one=False)),
    "the gate is a silu": ("dense_ff", _ff(plain=True)),
    "there is one norm": ("layer", _one_norm),
    "the feed-forward reads the mixer's sum": ("layer", _in_series),
    "a pass begins with the residual alone": ("enter_pass", lambda x, x0, W, t, f=O.enter_pass: f(x, 0 * x0, W, t)),
    "every pass has the first one's step": ("enter_pass", lambda x, x0, W, t, f=O.enter_pass: f(x, x0, W, 0)),
    "only the first pass is entered": ("enter_pass", lambda x, x0, W, t, f=O.enter_pass: f(x, x0, W, t) if t == 0 else x),
}


@pytest.mark.parametrize("mistake", MISTAKES)
def test_weights_show_mistakes(mistake, monkeypatch):
    """The tests' weights make each mistake visible well above what bf16 rounding does (test_bibapel_gpu.WHOLE)."""
    cfg = S.CONFIGS["uneven"]
    W, toks = S.make_weights(cfg), S.tokens(72, cfg["vocab"], 5)
    good = O.forward(cfg, W, toks)
    monkeypatch.setattr(O, *MISTAKES[mistake])
    e = S.error(O.forward(cfg, W, toks), good)
    print(mistake, round(e, 3))
    assert e > 0.12


def test_bench_option_parses():
    import bench
    assert bench.parse(["--stack", "all", "--stack-design", "bibapel"]).stack_design == "bibapel"
    from nats_llm_studio_amd import bench_stack
    for size in bench_stack.SIZES["bibapel"].values():
        c = StackConfig.from_json(bench_stack.CONFIGS["bibapel"](size))
        assert {L.mixer.kind for L in c.layers} == {"channel_delta", "attention", "lightning"}
