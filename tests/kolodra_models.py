"""Small random Kolodra models for the tests: configurations of several shapes and weights that keep every mechanism visible
in the logits."""
import torch

from sekolorn_models import error, tokens, write_model       # noqa: F401


def left(heads=6, kv_heads=2, dim=20, rot=12, base=700.0, scale=0.3):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "rot": {"base": base, "dims": rot}, "scale": scale}


def right(heads=3, dim=20, vdim=28, tau=7.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}


def layer(lf=None, rt=None, ff=72, left_scale=0.8, right_scale=1.3, weights_of=None):
    m = {"left": lf or left(), "right": rt or right(), "left_scale": left_scale, "right_scale": right_scale}
    d = {"type": "parallel", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}
    if weights_of is not None:
        d["weights_of"] = weights_of
    return d


def config(layers, width=136, vocab=203, eps=3e-5, embed=3.0, cap=9.0):
    return {"architecture": "Kolodra", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers,
            "embedding": {"scale": embed}, "logit_softcap": cap}


_plain = layer(ff=0, left_scale=1.1, right_scale=0.7)
# name -> config: uneven sizes and shared weights, one-of-everything sizes, sizes past the kernels' tiles (more than 16 query
# heads per key head, wide keys and values), head widths without an MFMA kernel and odd value widths
CONFIGS = {
    "uneven": config([layer(), _plain, layer(weights_of=0), layer(left(3, 3, 34, 34), right(2, 33, 16, 2.0), 50),
                      dict(_plain, weights_of=1), layer(weights_of=2)]),
    "ones": config([layer(left(1, 1, 8, 2, 40.0, 1.0), right(1, 4, 4, 1.0), 16, 1.0, 1.0)], width=48, vocab=37, eps=1e-6,
                   embed=1.0, cap=30.0),
    "wide": config([layer(left(40, 2, 64, 32, 1e4, 0.11), right(3, 130, 96, 16.0), 384),
                    layer(left(10, 10, 32, 32, 1e4, 0.2), right(5, 64, 136, 4.0), 130, -0.6, 1.0)], width=320, vocab=515),
    "big heads": config([layer(left(3, 1, 200, 64, 1e4, 0.06), right(1, 256, 264, 9.0), 40),
                         layer(left(2, 1, 128, 128, 1e4, 0.09), right(2, 16, 512, 5.0), 40)], width=72),
    "odd": config([layer(left(2, 1, 300, 100, 500.0, 0.05), right(2, 30, 21, 3.0), 36),
                   layer(left(5, 5, 33, 0, 1.0, 0.2), right(1, 7, 5, 3.0), 2)], width=90, vocab=101),
}


def make_weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    W = {}

    def lin(name, out, inp, gain=1.0):
        W[name] = (torch.randn(out, inp, generator=g) * gain * inp ** -0.5).to(torch.bfloat16)

    def near(name, n, mid):
        W[name] = (mid + 0.3 * torch.randn(n, generator=g)).to(torch.bfloat16)

    d = cfg["width"]
    W["embed"] = (torch.randn(cfg["vocab"], d, generator=g) / cfg["embedding"]["scale"]).to(torch.bfloat16)
    for i, L in enumerate(cfg["layers"]):
        if L.get("weights_of") is not None:
            continue
        p, a, r = f"l{i}.", L["mixer"]["left"], L["mixer"]["right"]
        near(p + "norm1", d, 0.0)
        q = p + "mix.left."
        H, G, D = a["heads"], a["kv_heads"], a["dim"]
        lin(q + "q", H * D, d)
        lin(q + "k", G * D, d)
        near(q + "q.norm", H * D, 1.3)
        near(q + "k.norm", G * D, 1.3)
        lin(q + "g", H, d, 1.5)
        lin(q + "o", d, H * D, 1.5)
        q = p + "mix.right."
        H, D, V, R = r["heads"], r["dim"], r["vdim"], 6 + 5 * i
        for n, rows in (("q", H * D), ("k", H * D), ("v", H * V), ("g", H * V)):
            lin(q + n, rows, d)
        lin(q + "a1", R, d)
        lin(q + "a2", H * D, R)
        W[q + "a2.b"] = (torch.rand(H * D, generator=g) * 8.0 - 4.0).to(torch.bfloat16)      # fast to slow decays
        near(q + "norm", V, 1.0)
        lin(q + "o", d, H * V)
        if L.get("mlp"):
            ff = L["mlp"]["ff"]
            lin(p + "mlp.gate", ff, d)
            lin(p + "mlp.up", ff, d)
            lin(p + "mlp.down", d, ff)
    near("final.norm", d, 0.0)
    lin("head", cfg["vocab"], d, 3.0)
    return W
