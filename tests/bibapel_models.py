"""Small random Bibapel models for the tests: configurations of several shapes and weights that keep every mechanism visible
in the logits."""
import torch

from sekolorn_models import error, tokens, write_model       # noqa: F401


def delta(heads=4, kv_heads=2, dim=20, vdim=28, conv=4):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def attention(heads=6, kv_heads=2, dim=20, vdim=36, scale=0.3, size=37, keep=5):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if size:
        m["mask"] = {"size": size, "keep_first": keep}
    return {"type": "attention", "mixer": m}


def lightning(decay=(0.5, 0.93, 0.995), dim=20, vdim=12):
    return {"type": "lightning", "mixer": {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}}


def layer(mixer, ff=72, limit=0.8):
    return dict(mixer, mlp={"kind": "dense", "ff": ff, "limit": limit} if ff else None)


def config(layers, width=136, vocab=203, eps=3e-5, scale=0.7, loop=None, buckets=67, mul=(13, 5), positions=1200):
    c = {"architecture": "Bibapel", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers,
         "embedding": {"scale": scale, "bigram": {"buckets": buckets, "mul_prev": mul[0], "mul_cur": mul[1]}},
         "max_positions": positions}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


# name -> config: uneven sizes with a loop in the middle, one-of-everything sizes in one pass, sizes past the kernels' tiles with a
# loop that ends the model, head widths without an MFMA kernel and odd sizes without a loop, no window and no recurrent mixer,
# products long enough to be split
CONFIGS = {
    "uneven": config([layer(lightning(), 0), layer(delta()), layer(attention()), layer(lightning((0.8, 0.99), 33, 28), 50, 1.4),
                      layer(attention(3, 3, 34, 20, 0.25, 16, 0), 0), layer(delta(3, 3, 33, 16, 2), 40)], loop=(1, 4, 3)),
    "ones": config([layer(delta(1, 1, 8, 16, 1), 16), layer(attention(1, 1, 8, 8, 1.0, 1, 1), 16), layer(lightning((0.9,), 4, 16), 16)],
                   width=48, vocab=37, eps=1e-6, scale=1.0, loop=(0, 3, 1), buckets=1, mul=(1, 1)),
    "wide": config([layer(attention(40, 2, 64, 64, 0.11, 130, 33), 384), layer(delta(6, 2, 130, 136, 3), 130),
                    layer(lightning((0.6, 0.9, 0.95, 0.99, 1.0), 64, 264), 0), layer(delta(2, 1, 64, 64, 4), 64, 7.0)],
                   width=320, vocab=515, loop=(2, 4, 2), mul=(30011, 70001), buckets=1009),
    "big heads": config([layer(attention(3, 1, 200, 130, 0.06, 64, 64), 40), layer(delta(1, 1, 256, 260, 5), 40),
                         layer(lightning((0.97,), 256, 512), 40)], width=72, loop=(0, 1, 2)),
    "odd": config([layer(attention(2, 1, 300, 10, 0.05, 20, 3), 36), layer(delta(2, 1, 30, 21, 3), 2),
                   layer(attention(5, 5, 33, 47, 0.2, 50, 17), 34), layer(lightning((0.2, 0.96), 7, 13), 6)], width=90, vocab=101),
    "attention only": config([layer(attention(4, 2, 24, 24, 0.3, 0)), layer(attention(4, 4, 16, 32, 0.4, 7, 40), 30)], width=64,
                             loop=(1, 2, 2)),
    "split": config([layer(attention(2, 1, 32, 32, 0.2, 40, 4), 40), layer(lightning((0.9, 0.97), 16, 24), 2090, 2.0)], width=1030,
                    vocab=101, loop=(0, 2, 2)),
}


def make_weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    W = {}

    def rnd(name, *shape, gain=1.0, mid=0.0):
        W[name] = (mid + torch.randn(*shape, generator=g) * gain).to(torch.bfloat16)

    def lin(name, out, inp, gain=1.0):
        rnd(name, out, inp, gain=gain * inp ** -0.5)

    def between(name, n, lo, hi):
        W[name] = (lo + (hi - lo) * torch.rand(n, generator=g)).to(torch.bfloat16)

    d, e = cfg["width"], cfg["embedding"]
    rnd("embed", cfg["vocab"], d)
    rnd("bigram", e["bigram"]["buckets"] + 1, d, gain=0.7)
    rnd("pos", cfg["max_positions"], d, gain=0.5)
    if cfg.get("loop"):
        lin("loop.in", d, 2 * d, 1.4)
        rnd("loop.step", cfg["loop"]["times"], d, gain=0.7)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        q = p + "mix."
        rnd(p + "norm1", d, gain=0.3, mid=1.0)
        H, D, V = m["heads"], m["dim"], m["vdim"]
        if L["type"] == "channel_delta":
            G, ra, rg = m["kv_heads"], 6 + 5 * i, 9 + 3 * i
            for n, rows in (("q", G * D), ("k", G * D), ("v", H * V)):
                lin(q + n, rows, d, 1.4)
                rnd(q + n + ".conv", rows, m["conv"], gain=0.5)
                W[q + n + ".conv"][:, -1] += 0.5
            lin(q + "b", H, d, 1.5)
            between(q + "A_log", H, -2.0, 1.0)
            lin(q + "a1", ra, d)
            lin(q + "a2", H * D, ra)
            between(q + "dt_bias", H * D, -5.0, 1.5)                     # slow to fast decays
            rnd(q + "norm", V, gain=0.3, mid=1.0)
            lin(q + "g1", rg, d, 1.5)
            lin(q + "g2", H * V, rg, 1.5)
            lin(q + "o", d, H * V, 1.5)
        elif L["type"] == "attention":
            G = m["kv_heads"]
            for n, rows, gain in (("q", H * D, 1.3), ("k", G * D, 1.3), ("v", G * V, 1.0)):
                lin(q + n, rows, d, gain)
            lin(q + "o", d, H * V, 2.0)
        else:
            for n, rows in (("q", H * D), ("k", H * D), ("v", H * V), ("g", H * V)):
                lin(q + n, rows, d, 1.5)
            rnd(q + "norm", H * V, gain=0.3, mid=1.0)
            lin(q + "o", d, H * V, 1.5)
        if L.get("mlp"):
            ff = L["mlp"]["ff"]
            rnd(p + "norm2", d, gain=0.3, mid=1.0)
            lin(p + "mlp.gate", ff, d, 1.5)
            lin(p + "mlp.up", ff, d, 1.5)
            lin(p + "mlp.down", d, ff, 1.5)
    rnd("final.norm", d, gain=0.3, mid=1.0)
    return W
