"""Small random Sekolorn models for the tests: configurations of several shapes and weights that keep every mechanism
visible in the logits."""
import json
import os

import torch


def mixer_wkv(heads=3, dim=20):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim}}


def mixer_latent(heads=5, dim=24, rot=12, vdim=20, kv_rank=40, q_rank=56, base=900.0, scale=0.21, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
         "rot": {"base": base, "dims": rot}, "scale": scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m}


def moe(experts=12, top=3, ff=40, groups=(3, 2), scale=1.7, shared=56):
    d = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "scale": scale}}
    if groups:
        d["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared:
        d["shared"] = {"ff": shared}
    return d


def config(layers, width=136, vocab=203, eps=3e-5):
    return {"architecture": "Sekolorn", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers}


def layer(mixer, mlp=None):
    return dict(mixer, mlp=mlp)


# name -> config: uneven sizes, one-of-everything sizes, sizes that are multiples of the kernels' tiles, orders
CONFIGS = {
    "uneven": config([layer(mixer_latent(), moe()), layer(mixer_wkv(), moe(experts=5, top=2, groups=None, shared=0)),
                      layer(mixer_latent(kv_from=0, heads=3, dim=16, vdim=28, q_rank=33, scale=0.3), None),
                      layer(mixer_wkv(2, 33), moe(experts=8, top=1, ff=24, groups=(4, 1)))]),
    "ones": config([layer(mixer_wkv(1, 16), moe(experts=1, top=1, ff=16, groups=(1, 1), scale=1.0, shared=16)),
                    layer(mixer_latent(1, 8, 2, 4, 8, 8, base=40.0, scale=1.0), moe(experts=2, top=2, ff=8, groups=(1, 1)))],
                   width=48, vocab=37, eps=1e-6),
    "wide": config([layer(mixer_wkv(3, 128), moe(experts=18, top=4, ff=64, groups=(6, 3), shared=128)),
                    layer(mixer_latent(18, 64, 64, 64, 192, 160, base=1e4, scale=0.09), moe(experts=32, top=6, ff=128)
                          | {"router": {"experts": 32, "top": 6, "scale": 2.0, "groups": {"count": 8, "keep": 4}}}),
                    layer(mixer_latent(17, 32, 64, 96, 192, 128, base=1e4, scale=0.11, kv_from=1), moe())],
                   width=320, vocab=515),
    "attention only": config([layer(mixer_latent(kv_rank=264, rot=70, heads=4), moe()), layer(mixer_latent(), None)],
                             width=96),
}


def make_weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    W = {}

    def rnd(name, *shape, gain=1.0):
        W[name] = (torch.randn(*shape, generator=g) * gain).to(torch.bfloat16)

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
    E = max([L["mlp"]["router"]["experts"] for L in cfg["layers"] if L.get("mlp")], default=0)
    levels = torch.linspace(-3.0, 3.0, max(E, 2))[:E]
    for t in range(cfg["vocab"]):
        W["embed"][t, :E] = levels[torch.randperm(E, generator=g)].to(torch.bfloat16)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        norm(p + "norm1", d, E)
        if L["type"] == "wkv":
            HD = m["heads"] * m["dim"]
            low = 8 + 4 * i
            for s in "rkvgw":
                W[p + "mix.mu." + s] = torch.rand(d, generator=g).to(torch.bfloat16)
            for s in "rkvg":
                lin(p + "mix." + s, HD, d, 0.7)
            lin(p + "mix.w1", low, d)
            lin(p + "mix.w2", HD, low)
            W[p + "mix.w0"] = (torch.rand(HD, generator=g) * 7.0 - 6.0).to(torch.bfloat16)      # slow to fast decays
            rnd(p + "mix.u", m["heads"], m["dim"], gain=0.5)
            norm(p + "mix.norm", HD)
            lin(p + "mix.o", d, HD)
        else:
            H, D, RD, VD, R, Q = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank"))
            lin(p + "mix.dq", Q, d)
            norm(p + "mix.dq.norm", Q)
            lin(p + "mix.uq", H * (D + RD), Q, 1.6)
            if "kv_from" not in m:
                lin(p + "mix.dkv", R + RD, d)
                norm(p + "mix.dkv.norm", R)
            lin(p + "mix.uk", H * D, R, 1.6)
            lin(p + "mix.uv", H * VD, R)
            lin(p + "mix.g", H, d)
            lin(p + "mix.o", d, H * VD)
        f = L.get("mlp")
        if f:
            norm(p + "norm2", d, E)
            n = f["router"]["experts"]
            lin(p + "mlp.router", n, d, 0.02)
            W[p + "mlp.router"][:, :n] += torch.eye(n).to(torch.bfloat16)[torch.randperm(n, generator=g)]
            for e in range(n):
                lin(f"{p}mlp.e{e}.up", f["expert"]["ff"], d)
                lin(f"{p}mlp.e{e}.down", d, f["expert"]["ff"])
            if f.get("shared"):
                lin(p + "mlp.shared.up", f["shared"]["ff"], d)
                lin(p + "mlp.shared.down", d, f["shared"]["ff"])
    norm("final.norm", d)
    lin("head", cfg["vocab"], d)
    return W


def write_model(path, cfg, W):
    from nats_llm_studio_amd.safetensors_io import write_safetensors
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_safetensors(os.path.join(path, "model.safetensors"), W)
    return path


def tokens(n, vocab, seed=1):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def error(got, want, q=1.0):
    """Row errors: rms over the vocabulary of the mean-free difference, over the rms of the wanted rows; their q-quantile
    (1: the largest)."""
    got, want = got.double(), want.double()
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    return float(torch.quantile(d.pow(2).mean(-1).sqrt() / (want - want.mean(-1, keepdim=True)).pow(2).mean().sqrt(), q))
