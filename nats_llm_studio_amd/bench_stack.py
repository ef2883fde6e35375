"""`bench.py --stack`: prefill and decode throughput of the config-driven stack designs at sizes of real layers, each beside the
GGUF families' closest model with the same width, layers and weights per layer, F16:
  sekolorn   Mixtral (attention + routed experts), the same experts
  kolodra    Llama (grouped-query attention + gated feed-forward), the feed-forward wider by the weights of the second mixer
  bibapel    Llama, four layers beside four layer runs (the attention layer runs twice), the feed-forward wider by the weights that
             the linear mixers and the passes' entries read
  pimodra    Mixtral, four layers beside four layer runs (one with a dense feed-forward of a token's expert weights, then experts,
             one of these layers twice), the same experts

Both run the engine's own loop: submit, chunked prefill, captured decode steps. Random weights; one JSON line per case."""
from __future__ import annotations

import json
import os
import time
from dataclasses import replace

VOCAB = 32000

# design -> size -> (its config arguments, closest model's arguments)
SIZES = {
    # expert weights: 2 * ff_s = 3 * ff_m
    "sekolorn": {
        "2k": dict(width=2048, wkv=(32, 64), latent=dict(heads=16, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=768),
                   moe=(8, 2, 6144), closest=dict(n_head=16, n_kv_head=4, d_ff=4096)),
        "4k": dict(width=4096, wkv=(64, 64), latent=dict(heads=32, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=1536),
                   moe=(8, 2, 6144), closest=dict(n_head=32, n_kv_head=8, d_ff=4096)),
        # many small experts, a shared one, group-limited choice (no GGUF family has this shape)
        "4k-fine": dict(width=4096, wkv=(64, 64), latent=dict(heads=32, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=1536),
                        moe=(64, 6, 1024), groups=(8, 4), shared=1024, closest=None),
    },
    "kolodra": {
        "2k": dict(width=2048, left=(16, 4, 128), right=(16, 64, 128), ff=5632, closest=dict(n_head=16, n_kv_head=4, d_ff=8192)),
        "4k": dict(width=4096, left=(32, 8, 128), right=(32, 64, 128), ff=9216, closest=dict(n_head=32, n_kv_head=8, d_ff=14336)),
    },
    # delta: heads, query and key heads, key and value width, rank of its gates; lightning: heads, key and value width
    "bibapel": {
        "2k": dict(width=2048, attention=(16, 4, 128), delta=(16, 8, 128, 128, 128), lightning=(16, 128, 128), ff=5632,
                   closest=dict(n_head=16, n_kv_head=4, d_ff=6912)),
        "4k": dict(width=4096, attention=(32, 8, 128), delta=(32, 16, 128, 128, 128), lightning=(32, 128, 128), ff=9216,
                   closest=dict(n_head=32, n_kv_head=8, d_ff=12288)),
    },
    # dense ff: 2 matrices = the 3 matrices of a token's experts
    "pimodra": {
        "2k": dict(width=2048, attention=(16, 4, 128), ff=12288, moe=(8, 2, 4096), closest=dict(n_head=16, n_kv_head=4, d_ff=4096)),
        "4k": dict(width=4096, attention=(32, 8, 128), ff=12288, moe=(8, 2, 4096), closest=dict(n_head=32, n_kv_head=8, d_ff=4096)),
        # many small experts, group-limited choice (no GGUF family has this shape)
        "4k-fine": dict(width=4096, attention=(32, 8, 128), ff=12288, moe=(64, 6, 1024), groups=(8, 4), closest=None),
    },
}
CLOSEST = {"sekolorn": "mixtral-8x7b", "kolodra": "llama-3-8b", "bibapel": "llama-3-8b", "pimodra": "mixtral-8x7b"}

def sekolorn_config(sz: dict) -> dict:
    H, D = sz["wkv"]
    lat = dict(sz["latent"], rot={"base": 10000.0, "dims": sz["latent"]["rot_dim"]}, scale=192 ** -0.5)
    E, top, ff = sz["moe"]
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": E, "top": top, "scale": 1.0}}
    if "groups" in sz:
        mlp["router"]["groups"] = {"count": sz["groups"][0], "keep": sz["groups"][1]}
    if "shared" in sz:
        mlp["shared"] = {"ff": sz["shared"]}
    layers = [{"type": "wkv", "mixer": {"heads": H, "dim": D}, "mlp": mlp}]
    layers += [{"type": "latent_attention", "mixer": dict(lat, **kv), "mlp": mlp} for kv in ({}, {}, {"kv_from": 2})]
    return {"architecture": "Sekolorn", "width": sz["width"], "vocab": VOCAB, "norm": {"eps": 1e-5}, "layers": layers}


def kolodra_config(sz: dict) -> dict:
    H, G, D = sz["left"]
    RH, RD, RV = sz["right"]
    mixer = {"left": {"heads": H, "kv_heads": G, "dim": D, "vdim": D, "rot": {"base": 10000.0, "dims": D}, "scale": D ** -0.5},
             "right": {"heads": RH, "dim": RD, "vdim": RV, "tau": 16.0}, "left_scale": 1.0, "right_scale": 1.0}
    layers = [{"type": "parallel", "mixer": mixer, "mlp": {"kind": "dense", "ff": sz["ff"]}} for _ in range(4)]
    return {"architecture": "Kolodra", "width": sz["width"], "vocab": VOCAB, "norm": {"eps": 1e-5}, "layers": layers,
            "embedding": {"scale": 1.0}, "logit_softcap": 30.0}


def bibapel_config(sz: dict) -> dict:
    H, G, D = sz["attention"]
    DH, DG, DD, DV, _ = sz["delta"]
    LH, LD, LV = sz["lightning"]
    mixers = [("channel_delta", {"heads": DH, "kv_heads": DG, "dim": DD, "vdim": DV, "conv": 4}),
              ("attention", {"heads": H, "kv_heads": G, "dim": D, "vdim": D, "scale": D ** -0.5,
                             "mask": {"size": 1024, "keep_first": 16}}),
              ("lightning", {"heads": LH, "dim": LD, "vdim": LV, "decay": [1.0 - 2.0 ** (-1 - 8 * h / LH) for h in range(LH)]})]
    layers = [{"type": t, "mixer": m, "mlp": {"kind": "dense", "ff": sz["ff"], "limit": 7.0}} for t, m in mixers]
    return {"architecture": "Bibapel", "width": sz["width"], "vocab": VOCAB, "norm": {"eps": 1e-5}, "layers": layers,
            "embedding": {"scale": 1.0, "bigram": {"buckets": 8191, "mul_prev": 127, "mul_cur": 3}}, "max_positions": 8192,
            "loop": {"start": 1, "stop": 2, "times": 2}, "rank": sz["delta"][4]}


def pimodra_config(sz: dict) -> dict:
    H, G, D = sz["attention"]
    E, top, ff = sz["moe"]
    mixer = {"heads": H, "kv_heads": G, "dim": D, "vdim": D, "scale": D ** -0.5, "mask": {"size": 1024},
             "rot": {"base": 10000.0, "dims": D, "scaling": {"factor": 4.0, "original": 2048, "fast": 32.0, "slow": 1.0}}}
    moe = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": E, "top": top}}
    if "groups" in sz:
        moe["router"]["groups"] = {"count": sz["groups"][0], "keep": sz["groups"][1]}
    layers = [{"type": "attention", "mixer": mixer, "mlp": f} for f in ({"kind": "dense", "ff": sz["ff"]}, moe, moe)]
    return {"architecture": "Pimodra", "width": sz["width"], "vocab": VOCAB, "norm": {"eps": 1e-5, "groups": 2}, "layers": layers,
            "loop": {"start": 1, "stop": 2, "times": 2}}


CONFIGS = {"sekolorn": sekolorn_config, "kolodra": kolodra_config, "bibapel": bibapel_config, "pimodra": pimodra_config}


def _sekolorn_layer(p: str, L: dict, d: int, lin, full):
    m = L["mixer"]
    full(p + "norm1", 1.0, d)
    full(p + "norm2", 1.0, d)
    if L["type"] == "wkv":
        HD = m["heads"] * m["dim"]
        for s in "rkvgw":
            full(p + "mix.mu." + s, 0.5, d)
        for s in "rkvg":
            lin(p + "mix." + s, HD, d)
        lin(p + "mix.w1", 64, d)
        lin(p + "mix.w2", HD, 64)
        full(p + "mix.w0", -3.0, HD)
        full(p + "mix.u", 0.5, m["heads"], m["dim"])
        full(p + "mix.norm", 1.0, HD)
        lin(p + "mix.o", d, HD)
    else:
        H, D, RD, VD, R, Q = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank"))
        lin(p + "mix.dq", Q, d)
        full(p + "mix.dq.norm", 1.0, Q)
        lin(p + "mix.uq", H * (D + RD), Q)
        if "kv_from" not in m:
            lin(p + "mix.dkv", R + RD, d)
            full(p + "mix.dkv.norm", 1.0, R)
        lin(p + "mix.uk", H * D, R)
        lin(p + "mix.uv", H * VD, R)
        lin(p + "mix.g", H, d)
        lin(p + "mix.o", d, H * VD)
    f = L["mlp"]
    lin(p + "mlp.router", f["router"]["experts"], d)
    for e in range(f["router"]["experts"]):
        lin(f"{p}mlp.e{e}.up", f["expert"]["ff"], d)
        lin(f"{p}mlp.e{e}.down", d, f["expert"]["ff"])
    if f.get("shared"):
        lin(p + "mlp.shared.up", f["shared"]["ff"], d)
        lin(p + "mlp.shared.down", d, f["shared"]["ff"])


def _kolodra_layer(p: str, L: dict, d: int, lin, full):
    a, r, ff = L["mixer"]["left"], L["mixer"]["right"], L["mlp"]["ff"]
    full(p + "norm1", 0.0, d)
    q = p + "mix.left."
    for n, rows in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"])):
        lin(q + n, rows, d)
        full(q + n + ".norm", 1.0, rows)
    lin(q + "g", a["heads"], d)
    lin(q + "o", d, a["heads"] * a["dim"])
    q, HD, HV = p + "mix.right.", r["heads"] * r["dim"], r["heads"] * r["vdim"]
    for n, rows in (("q", HD), ("k", HD), ("v", HV), ("g", HV)):
        lin(q + n, rows, d)
    lin(q + "a1", 16, d)
    lin(q + "a2", HD, 16)
    full(q + "a2.b", 1.0, HD)
    full(q + "norm", 1.0, r["vdim"])
    lin(q + "o", d, HV)
    lin(p + "mlp.gate", ff, d)
    lin(p + "mlp.up", ff, d)
    lin(p + "mlp.down", d, ff)


def _bibapel_layer(p: str, L: dict, d: int, lin, full, rank: int):
    m, ff = L["mixer"], L["mlp"]["ff"]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    full(p + "norm1", 1.0, d)
    full(p + "norm2", 1.0, d)
    q = p + "mix."
    if L["type"] == "channel_delta":
        for n, rows in (("q", m["kv_heads"] * D), ("k", m["kv_heads"] * D), ("v", H * V)):
            lin(q + n, rows, d)
            lin(q + n + ".conv", rows, m["conv"])
        lin(q + "b", H, d)
        full(q + "A_log", 0.0, H)
        lin(q + "a1", rank, d)
        lin(q + "a2", H * D, rank)
        full(q + "dt_bias", -3.0, H * D)
        full(q + "norm", 1.0, V)
        lin(q + "g1", rank, d)
        lin(q + "g2", H * V, rank)
    elif L["type"] == "attention":
        for n, rows in (("q", H * D), ("k", m["kv_heads"] * D), ("v", m["kv_heads"] * V)):
            lin(q + n, rows, d)
    else:
        for n, rows in (("q", H * D), ("k", H * D), ("v", H * V), ("g", H * V)):
            lin(q + n, rows, d)
        full(q + "norm", 1.0, H * V)
    lin(q + "o", d, H * V)
    lin(p + "mlp.gate", ff, d)
    lin(p + "mlp.up", ff, d)
    lin(p + "mlp.down", d, ff)


def _pimodra_layer(p: str, L: dict, d: int, lin, full):
    m, f = L["mixer"], L["mlp"]
    for n in ("norm1", "norm1b", "norm2", "norm2b"):
        full(p + n, 1.0, d)
    H, G, D, V = (m[k] for k in ("heads", "kv_heads", "dim", "vdim"))
    for n, rows in (("q", H * D), ("k", G * D), ("v", G * V), ("g", H * V)):
        lin(p + "mix." + n, rows, d)
    lin(p + "mix.talk", H, H)
    lin(p + "mix.o", d, H * V)
    if f["kind"] == "dense":
        lin(p + "mlp.up", f["ff"], d)
        lin(p + "mlp.down", d, f["ff"])
        full(p + "mlp.act", 0.5, 4)
        return
    lin(p + "mlp.router", f["router"]["experts"], d)
    for e in range(f["router"]["experts"]):
        for n in ("gate", "up"):
            lin(f"{p}mlp.e{e}.{n}", f["expert"]["ff"], d)
        lin(f"{p}mlp.e{e}.down", d, f["expert"]["ff"])


def write_stack(path: str, cfg: dict):
    """A checkpoint folder of `cfg` with random weights."""
    import torch

    from .models.stack_config import DESIGNS
    from .safetensors_io import write_safetensors
    os.makedirs(path, exist_ok=True)
    W, d = {}, cfg["width"]
    dev = "cuda" if torch.cuda.is_available() else "cpu"
    g = torch.Generator(device=dev).manual_seed(0)

    def lin(name, *shape):
        W[name] = (torch.randn(*shape, generator=g, device=dev) * shape[-1] ** -0.5).to(torch.bfloat16).cpu()

    def full(name, v, *shape):
        W[name] = torch.full(shape, v, dtype=torch.bfloat16)
    W["embed"] = torch.randn(cfg["vocab"], d, generator=g, device=dev).to(torch.bfloat16).cpu()
    layer = {"Sekolorn": _sekolorn_layer, "Kolodra": _kolodra_layer, "Bibapel": _bibapel_layer,
             "Pimodra": _pimodra_layer}[cfg["architecture"]]
    cfg = dict(cfg)
    rank = cfg.pop("rank", None)                    # (of the delta rule's gates: a tensor shape, no part of the config)
    for i, L in enumerate(cfg["layers"]):
        layer(f"l{i}.", L, d, lin, full, *([] if rank is None else [rank]))
    full("final.norm", 0.0 if cfg["architecture"] == "Kolodra" else 1.0, d)
    if cfg["architecture"] == "Bibapel":
        lin("bigram", cfg["embedding"]["bigram"]["buckets"] + 1, d)
        lin("pos", cfg["max_positions"], d)
        lin("loop.in", d, 2 * d)
    if cfg.get("loop"):
        lin("loop.step", cfg["loop"]["times"], d)
    if not DESIGNS[cfg["architecture"]].tied_head:
        lin("head", cfg["vocab"], d)
    with open(os.path.join(path, "config.json"), "w") as fh:
        json.dump(cfg, fh)
    write_safetensors(os.path.join(path, "model.safetensors"), W)


def load(design: str, closest: bool, size: str, model_dir: str, dev):
    from .models.registry import load_model
    sz = SIZES[design][size]
    os.makedirs(model_dir, exist_ok=True)
    if not closest:
        path = os.path.join(model_dir, f"{design}-{size}")
        if not os.path.exists(os.path.join(path, "config.json")):
            write_stack(path, CONFIGS[design](sz))
        return load_model(path, dev, ctx=8192)
    from .gguf import synth
    # F16 weights run on the dense GEMMs' row-major copies (the LDS-dequant GEMM takes K-quants only)
    os.environ.setdefault("NLS_DENSE_WEIGHTS", "1")
    os.environ.setdefault("NLS_DENSE_EXPERTS", "1")
    name = f"{CLOSEST[design].split('-')[0]}-{size}"
    path = os.path.join(model_dir, f"{name}.gguf")
    if not os.path.exists(path):
        moe = dict(n_expert=sz["moe"][0], n_expert_used=sz["moe"][1]) if "moe" in sz else {}
        synth.SPECS[name] = replace(synth.SPECS[CLOSEST[design]], name=name, n_layer=4, d_model=sz["width"], vocab=VOCAB,
                                    **moe, **sz["closest"])
        synth.write_synthetic_gguf(path, name, "F16", seed=0)
    return load_model(path, dev)


def measure(model, B: int, prompt: int, steps: int, warmup: int, repeat: int = 2) -> dict:
    """Prefill of B prompts (the last repeat is reported), then `steps` decode steps of the B sequences."""
    import numpy as np
    import torch

    from .engine.engine import Engine, GenRequest
    from .engine.sampling import SamplingParams
    rng = np.random.default_rng(0)
    eng = Engine(model, None, max_batch=B, max_prefill_tokens=4096, ctx=prompt + warmup + steps + 64,
                 num_blocks=(B + 1) * ((prompt + warmup + steps) // 16 + 4), prefix_cache=False)
    eng.capture_all([eng._bucket(B)])
    t_pre = t_dec = 0.0
    for r in range(repeat):
        futs = [eng.submit(GenRequest(list(rng.integers(0, VOCAB, prompt)), SamplingParams(
            max_tokens=warmup + steps + 12, ignore_eos=True))) for _ in range(B)]
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        while eng.waiting or any(s.n_prefilled < s.n_target for s in eng.running):
            eng._admit()
            eng._prefill()
        torch.cuda.synchronize()
        t_pre = time.perf_counter() - t0
        for _ in range(warmup):
            eng.step()
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        for _ in range(steps):
            eng.step()
        torch.cuda.synchronize()
        t_dec = time.perf_counter() - t0
        while not all(f.done() for f in futs):
            eng.step()
    eng.unload()
    return dict(prefill_tok_s=round(B * prompt / t_pre, 1), prefill_ms=round(t_pre * 1e3, 3),
                decode_tok_s=round(B * steps / t_dec, 1), decode_ms_per_step=round(t_dec / steps * 1e3, 4))


CASES = {"prefill": [(1, 512), (1, 4096), (8, 1024)], "decode": [(1, 1024), (16, 1024), (64, 1024), (256, 512)]}


def run(args) -> int:
    import torch
    dev = torch.device("cuda:0")
    cases = CASES["prefill"] + CASES["decode"] if args.stack == "all" else CASES[args.stack]
    if args.stack_case:
        cases = [tuple(int(v) for v in args.stack_case.split("x"))]
    design, sizes = args.stack_design, SIZES[args.stack_design]
    for size in [z for z in args.stack_sizes.split(",") if z in sizes]:
        for which in (design, "closest"):
            if args.stack_only not in (None, which) or (which == "closest" and sizes[size]["closest"] is None):
                continue
            t0 = time.time()
            model = load(design, which == "closest", size, args.model_dir, dev)
            t_load = time.time() - t0
            for B, prompt in cases:
                steps = 4 if (B, prompt) in CASES["prefill"] and args.stack != "decode" and not args.stack_case else args.steps
                out = measure(model, B, prompt, min(steps, 100), min(args.warmup, 10))
                print(json.dumps(dict(bench="stack", model=which, size=size, batch=B, prompt=prompt, layers=4,
                                      weights_gb=round(model.weight_bytes / 1e9, 3), load_s=round(t_load, 1),
                                      dtype="fp16" if which == "closest" else "bf16", data="synthetic", **out)), flush=True)
            del model
            torch.cuda.empty_cache()
    return 0
