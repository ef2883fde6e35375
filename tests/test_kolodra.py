"""Kolodra on the CPU: configuration, shared weights, and the plain implementation against itself (cut sequences, hand-computed
values, planted mistakes). The kernels are in test_kolodra_gpu.py."""
import json

import numpy as np
import pytest
import torch

import kolodra_models as S
import kolodra_oracle as O
from nats_llm_studio_amd.models.registry import checkpoint_kind, stack_arch, supported_architectures
from nats_llm_studio_amd.models.stack_config import StackConfig, weight_owners


def shapes(W):
    return lambda n: tuple(W[n].shape) if n in W else None


@pytest.mark.parametrize("name", S.CONFIGS)
def test_config(name):
    cfg = S.CONFIGS[name]
    W = S.make_weights(cfg)
    c = StackConfig.from_json(cfg, shapes(W))
    assert (c.d_model, c.vocab, c.eps, c.n_layer) == (cfg["width"], cfg["vocab"], cfg["norm"]["eps"], len(cfg["layers"]))
    assert (c.embed_scale, c.softcap, c.recurrent, c.n_expert) == (cfg["embedding"]["scale"], cfg["logit_softcap"], True, 0)
    for i, (L, l) in enumerate(zip(cfg["layers"], c.layers)):
        a, r, m = L["mixer"]["left"], L["mixer"]["right"], l.mixer
        assert (m.left.heads, m.left.kv_heads, m.left.dim, m.left.rot_dims, m.left.rot_base, m.left.scale) == (
            a["heads"], a["kv_heads"], a["dim"], a["rot"]["dims"], a["rot"]["base"], a["scale"])
        assert (m.right.heads, m.right.dim, m.right.vdim, m.right.tau) == (r["heads"], r["dim"], r["vdim"], r["tau"])
        assert (m.left_scale, m.right_scale) == (L["mixer"]["left_scale"], L["mixer"]["right_scale"])
        assert (l.mlp.ff if l.mlp else None) == (L["mlp"]["ff"] if L["mlp"] else None)
        assert (i if l.weights_of is None else l.weights_of) == O.owner(cfg, i)
    # sizes that the config leaves out come from the tensors
    lean = json.loads(json.dumps(cfg))
    for k in ("width", "vocab"):
        lean.pop(k)
    for L in lean["layers"]:
        for k in ("heads", "kv_heads", "dim", "vdim"):
            L["mixer"]["left"].pop(k)
        for k in ("heads", "dim", "vdim"):
            L["mixer"]["right"].pop(k)
        if L["mlp"]:
            L["mlp"].pop("ff")
    assert StackConfig.from_json(lean, shapes(W)) == c


def test_config_refusals():
    def bad(edit, exc=ValueError, name="uneven"):
        c = json.loads(json.dumps(S.CONFIGS[name]))
        edit(c)
        with pytest.raises(exc):
            StackConfig.from_json(c)
    bad(lambda c: c["layers"][0].update(type="wkv"), NotImplementedError)           # not a mixer of this design
    bad(lambda c: c["layers"][0]["mlp"].update(kind="moe"), NotImplementedError)
    bad(lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=4))               # 6 heads over 4
    bad(lambda c: c["layers"][3]["mixer"]["left"].update(vdim=35))                  # the values are the keys
    bad(lambda c: c["layers"][3]["mixer"]["left"]["rot"].update(dims=36))           # more than the head has
    bad(lambda c: c["layers"][3]["mixer"]["left"]["rot"].update(dims=7))
    bad(lambda c: c["layers"][2].update(weights_of=9))
    bad(lambda c: c["layers"][2].update(weights_of=2))                              # its own
    bad(lambda c: c["layers"][2]["mixer"].update(left_scale=0.5))                   # not its owner's entry
    bad(lambda c: c["layers"][2].update(mlp=None))


def test_weight_owners():
    of = lambda *w: weight_owners([{"weights_of": x} if x is not None else {} for x in w])      # noqa: E731
    assert of(None, None, 0, 2, 1) == [0, 1, 0, 0, 1] and of(1, None) == [1, 1] and of(None, 0, 0) == [0, 0, 0]
    with pytest.raises(ValueError):
        of(1, 0)


def test_registry(tmp_path):
    cfg = S.CONFIGS["ones"]
    d = S.write_model(str(tmp_path / "pub" / "Tiny-Kolo"), cfg, S.make_weights(cfg))
    assert checkpoint_kind(d) == "stack" and stack_arch(d) == "Kolodra" and "Kolodra" in supported_architectures()
    from nats_llm_studio_amd.service.registry import Registry
    reg = Registry(str(tmp_path))
    (e,) = reg.scan()
    assert e.id == "tiny-kolo" and e.arch == "Kolodra" and e.quantization == "BF16" and e.path == d


def test_launch_shapes():
    """Segments of the recurrence: at least 64 tokens each, none for decoding or for many runs."""
    from nats_llm_studio_amd.ops import stack as K
    for T, n, H, V in ((1, 1, 4, 64), (7, 7, 2, 20), (130, 3, 2, 64), (4096, 1, 32, 128), (4096, 4, 4, 512)):
        nseg, nt = K.gla_shape(T, n, H, V)
        assert 1 <= nseg <= 16 and (nseg == 1 or (T - n + 1) // nseg >= 64) and nt == (1 if V <= 64 else 2)
    assert K.gla_shape(4096, 1, 4, 64)[0] == 16 and K.gla_shape(4096, 8, 32, 128)[0] == 1
    assert K.head_pad(20) == (32, True) and K.head_pad(129) == (256, True) and K.head_pad(300) == (320, False)
    assert K.attn_groups(40, 2) == 4 and K.attn_groups(16, 1) == 1 and K.attn_groups(3, 3) == 3


# ---- the plain implementation against itself

def test_oracle_cut_sequences():
    """Both mixers fed in pieces, with carried keys and state, equal one pass."""
    cfg = S.CONFIGS["uneven"]
    W = {k: v.double() for k, v in S.make_weights(cfg).items()}
    eps, m = cfg["norm"]["eps"], cfg["layers"][0]["mixer"]
    h = torch.randn(23, cfg["width"], generator=torch.Generator().manual_seed(3), dtype=torch.float64)
    pos = torch.arange(23)
    whole, _ = O.parallel_mixer(h, W, "l0.mix.", m, pos, eps)
    before, out = None, []
    for a, b in ((0, 1), (1, 3), (3, 16), (16, 23)):
        y, before = O.parallel_mixer(h[a:b], W, "l0.mix.", m, pos[a:b], eps, before)
        out.append(y)
    assert torch.allclose(torch.cat(out), whole, atol=1e-10)


def test_oracle_known_values():
    """Hand-computed cases."""
    x = torch.tensor([[3.0, 4.0]])
    assert torch.allclose(O.norm_one_plus(x, torch.tensor([0.5, -1.0]), 0.5), x / 13.0 ** 0.5 * torch.tensor([1.5, 0.0]))
    r = O.rotate(torch.tensor([[[1.0, 0.0, 1.0, 0.0, 5.0]]], dtype=torch.float64), torch.tensor([2]), 100.0, 4)
    a = torch.tensor([2.0, 0.2], dtype=torch.float64)
    assert torch.allclose(r[0, 0], torch.cat([torch.stack([a.cos(), a.sin()], 1).reshape(-1), torch.tensor([5.0])]).double())
    one = lambda *v: torch.tensor(v, dtype=torch.float64).view(len(v), 1, 1)      # noqa: E731
    o, s = O.gla_scan(one(1.0, 2.0), one(2.0, 3.0), one(5.0, 7.0), one(0.1, 0.5))
    assert o.flatten().tolist() == [10.0, 52.0] and float(s) == 26.0
    z = torch.tensor([0.0, 10.0, -10.0], dtype=torch.float64)
    assert torch.allclose(O.gelu_tanh(z), torch.tensor([0.0, 10.0, 0.0], dtype=torch.float64), atol=1e-6)
    assert abs(float(O.softcap(torch.tensor(1e6), 9.0)) - 9.0) < 1e-5
    # a group's heads share their key head: 4 query heads, 2 key heads
    q, k = torch.zeros(1, 4, 1).double(), torch.zeros(1, 2, 1).double()
    v = torch.tensor([[[1.0], [2.0]]]).double()
    assert O.attend(q, k, v, torch.tensor([0]), 1.0).flatten().tolist() == [1.0, 1.0, 2.0, 2.0]


def _rows(f, values=None, drop=False):
    def g(h, W, p, m, positions, eps):
        q, k, v = f(h, W, p, m, positions, eps)
        if drop:
            k, v = (torch.cat([t[:7], t[6:7], t[8:]]) for t in (k, v))
        return q, k, k if values else v
    return g


def _heads_norm(h, W, p, m, positions, eps):
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    k0 = (h @ W[p + "k"].T).reshape(-1, G, D)
    q = O.rms((h @ W[p + "q"].T).reshape(-1, H, D), eps) * W[p + "q.norm"].view(H, D)
    k, r = O.rms(k0, eps) * W[p + "k.norm"].view(G, D), m["rot"]
    return O.rotate(q, positions, r["base"], r["dims"]), O.rotate(k, positions, r["base"], r["dims"]), k0


def _halves(x, positions, base, dims, f=O.rotate):
    n = dims // 2
    i = torch.stack([torch.arange(n), torch.arange(n) + n], 1).reshape(-1)
    y = f(torch.cat([x[..., i], x[..., dims:]], -1), positions, base, dims)
    return torch.cat([torch.cat([y[..., 0:dims:2], y[..., 1:dims:2]], -1), y[..., dims:]], -1)


def _read_first(q, k, v, a, state=None, f=O.gla_scan):
    """The state is read ahead of the token's update."""
    o, S = f(q, k, v, a, state)
    own = (q * k).sum(-1, keepdim=True) * v
    return o - own, S


def _values_decay(q, k, v, a, state=None, f=O.gla_scan):
    """The decay acts on the value columns (as far as there are any)."""
    n = min(a.shape[2], v.shape[2])
    w = torch.ones(v.shape).double()
    w[..., :n] = a[..., :n]
    S, out = torch.zeros(q.shape[1], q.shape[2], v.shape[2]).double(), []
    for t in range(q.shape[0]):
        S = w[t][:, None, :] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


MISTAKES = {
    "a key is missed": ("attention_rows", _rows(O.attention_rows, drop=True)),
    "the values are normed and rotated": ("attention_rows", _rows(O.attention_rows, values=True)),
    "queries and keys are normed per head": ("attention_rows", _heads_norm),
    "nothing is rotated": ("rotate", lambda x, *a: x),
    "halves are paired": ("rotate", _halves),
    "the whole head is rotated": ("rotate", lambda x, p, b, d, f=O.rotate: f(x, p, b, x.shape[-1] // 2 * 2)),
    "the first token is not seen": ("attend", lambda q, k, v, p, s, f=O.attend: torch.cat(
        [f(q[:1], k, v, p[:1], s), f(q[1:], k[1:], v[1:], p[1:] - 1, s)])),
    "the state is read before the update": ("gla_scan", _read_first),
    "the decay acts on the values": ("gla_scan", _values_decay),
    "there is no decay": ("decay", lambda *a, f=O.decay: torch.ones_like(f(*a))),
    "tau is left out": ("decay", lambda h, W, p, m, f=O.decay: f(h, W, p, dict(m, tau=1.0))),
    "the state is lost at token 20": ("gla_scan", lambda q, k, v, a, s=None, f=O.gla_scan: (torch.cat(
        [f(*(t[:20] for t in (q, k, v, a)))[0], f(*(t[20:] for t in (q, k, v, a)))[0]]), None)),
    "the logits are not capped": ("softcap", lambda z, c: z),
    "the norm's weight is not one-plus": ("norm_one_plus", lambda x, w, eps: O.rms(x, eps) * (1 + 0 * w)),
}


@pytest.mark.parametrize("mistake", MISTAKES)
def test_weights_show_mistakes(mistake, monkeypatch):
    """The tests' weights make each mistake visible well above what bf16 rounding does (test_kolodra_gpu.WHOLE)."""
    cfg = S.CONFIGS["uneven"]
    W, toks = S.make_weights(cfg), S.tokens(48, cfg["vocab"])
    good = O.forward(cfg, W, toks)
    monkeypatch.setattr(O, *MISTAKES[mistake])
    assert S.error(O.forward(cfg, W, toks), good) > 0.12


def test_bench_option_parses():
    import bench
    a = bench.parse([])
    assert a.stack is None and a.model == "llama-3-8b"
    assert bench.parse(["--stack", "all", "--stack-design", "kolodra"]).stack_design == "kolodra"
    assert bench.parse(["--stack", "decode"]).stack_design == "sekolorn" and np.prod(a.gpus) == 1
