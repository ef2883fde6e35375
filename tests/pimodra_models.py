"""Small random Pimodra models for the tests: configurations of several shapes and weights that keep every mechanism visible
in the logits."""
import torch

from sekolorn_models import error, tokens, write_model       # noqa: F401


def scaling(factor=3.0, original=300, fast=9.0, slow=0.6):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


def attention(heads=6, kv_heads=2, dim=20, vdim=36, scale=0.25, size=37, dims=12, base=900.0, yarn=scaling()):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": size}}
    if dims:
        m["rot"] = {"base": base, "dims": dims}
        if yarn:
            m["rot"]["scaling"] = yarn
    return m


def dense(ff=72):
    return {"kind": "dense", "ff": ff}


def moe(experts=10, top=3, ff=24, groups=(5, 3)):
    r = {"experts": experts, "top": top}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r}


def layer(mixer, mlp=None):
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def config(layers, width=136, vocab=203, eps=3e-5, groups=4, loop=None):
    c = {"architecture": "Pimodra", "width": width, "vocab": vocab, "norm": {"eps": eps, "groups": groups}, "layers": layers}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


# name -> config: uneven sizes with a loop in the middle, one-of-everything sizes in one pass, sizes past the kernels' tiles with a
# loop that ends the model (key heads that do not divide among the waves), head widths without an MFMA kernel and odd sizes
# without a loop, more heads than the prompt kernel takes, products long enough to be split with norm groups of whole waves
CONFIGS = {
    "uneven": config([layer(attention(), dense()), layer(attention(10, 5, 34, 20, 0.2, 16, 34), moe()), layer(attention(vdim=12)),
                      layer(attention(3, 3, 33, 33, 0.3, 5, 8, 50.0), moe(12, 2, 17, (3, 1))), layer(attention(size=90), dense(37))],
                     loop=(1, 4, 3)),
    "ones": config([layer(attention(1, 1, 8, 8, 1.0, 1, 2), moe(1, 1, 16, None)), layer(attention(2, 1, 4, 4, 0.7, 3, 4), dense(8))],
                   width=48, vocab=37, eps=1e-6, groups=1, loop=(0, 1, 1)),
    "wide": config([layer(attention(24, 2, 64, 64, 0.11, 130, 64), dense(384)), layer(attention(32, 32, 96, 128, 0.1, 64, 32), None),
                    layer(attention(20, 10, 128, 40, 0.08, 200, 128, 1e4, scaling(1.0, 64, 2.0, 1.0)), moe(16, 4, 64, (4, 2)))],
                   width=320, vocab=515, groups=5, loop=(1, 3, 2)),
    "big heads": config([layer(attention(3, 1, 200, 130, 0.06, 64, 200), dense(40)), layer(attention(2, 2, 300, 10, 0.05, 20, 6), moe())],
                        width=72, groups=3, loop=(0, 1, 2)),
    "odd": config([layer(attention(5, 5, 33, 47, 0.2, 50, 32, yarn=None), moe(7, 2, 9, None)),
                   layer(attention(7, 1, 15, 13, 0.3, 17, 0), dense(34))], width=90, vocab=101, groups=6),
    "many heads": config([layer(attention(40, 4, 32, 20, 0.2, 33, 32), dense(50)), layer(attention(70, 10, 20, 32, 0.25, 70, 20), moe())],
                         width=100, groups=2, loop=(1, 2, 2)),
    "split": config([layer(attention(4, 2, 32, 32, 0.2, 40, 32), dense(2090)), layer(attention(4, 4, 64, 64, 0.2, 600, 64), moe())],
                    width=1024, vocab=101, groups=4, loop=(0, 2, 2)),
}


def make_weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    W = {}

    def rnd(name, *shape, gain=1.0, mid=0.0):
        W[name] = (mid + torch.randn(*shape, generator=g) * gain).to(torch.bfloat16)

    def lin(name, out, inp, gain=1.0):
        rnd(name, out, inp, gain=gain * inp ** -0.5)

    def norm(name, n, quiet=0):
        w = 1.0 + 0.3 * torch.randn(n, generator=g)
        w[:quiet] *= 0.01
        W[name] = w.to(torch.bfloat16)

    d = cfg["width"]
    rnd("embed", cfg["vocab"], d)
    # Routing without close calls: the first columns of the residual hold evenly spaced levels in an order of the token's
    # own, the sublayers barely touch them (norm weights), and the routers read them.
    E = max([L["mlp"]["router"]["experts"] for L in cfg["layers"] if (L.get("mlp") or {}).get("kind") == "moe"], default=0)
    levels = torch.linspace(-2.0, 2.0, max(E, 2))[:E]
    for t in range(cfg["vocab"]):
        W["embed"][t, :E] = levels[torch.randperm(E, generator=g)].to(torch.bfloat16)
    if cfg.get("loop"):
        rnd("loop.step", cfg["loop"]["times"], d, gain=0.7)
        W["loop.step"][:, :E] = 0
    for i, L in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", L["mixer"], L.get("mlp")
        q = p + "mix."
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        norm(p + "norm1", d)
        norm(p + "norm1b", d, E)
        # (queries and keys end as unit vectors: what is large here is how far their directions turn with the token)
        for n, rows in (("q", H * D), ("k", G * D), ("v", G * V), ("g", H * V)):
            lin(q + n, rows, d, 1.5)
        lin(q + "talk", H, H)
        W[q + "talk"] += torch.eye(H).to(torch.bfloat16)
        lin(q + "o", d, H * V)
        if not f:
            continue
        norm(p + "norm2", d)
        norm(p + "norm2b", d, E)
        if f["kind"] == "dense":
            lin(p + "mlp.up", f["ff"], d)
            lin(p + "mlp.down", d, f["ff"])
            W[p + "mlp.act"] = torch.tensor([0.9, -0.6, 0.7, 0.4]).to(torch.bfloat16)
            continue
        n = f["router"]["experts"]
        W[p + "norm2"][:E] = 1.0
        lin(p + "mlp.router", n, d, 0.02)
        W[p + "mlp.router"][:, :n] += torch.eye(n).to(torch.bfloat16)[torch.randperm(n, generator=g)]
        for e in range(n):
            lin(f"{p}mlp.e{e}.gate", f["expert"]["ff"], d, 1.5)
            lin(f"{p}mlp.e{e}.up", f["expert"]["ff"], d, 1.5)
            lin(f"{p}mlp.e{e}.down", d, f["expert"]["ff"])
    norm("final.norm", d)
    return W
