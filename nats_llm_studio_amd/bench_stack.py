"""`bench.py --stack`: prefill and decode throughput of the Sekolorn design at sizes of real layers, beside the GGUF families'
closest model (Mixtral: attention + routed experts, F16 weights) with the same width, layers, experts and expert weights.

Both run the engine's own loop: submit, chunked prefill, captured decode steps. Random weights; one JSON line per case."""
from __future__ import annotations

import json
import os
import time
from dataclasses import replace

VOCAB = 32000

# name -> (Sekolorn config arguments, closest model's arguments); expert weights: 2 * ff_s = 3 * ff_m
SIZES = {
    "2k": dict(width=2048, wkv=(32, 64), latent=dict(heads=16, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=768),
               moe=(8, 2, 6144), mixtral=dict(n_head=16, n_kv_head=4, d_ff=4096)),
    "4k": dict(width=4096, wkv=(64, 64), latent=dict(heads=32, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=1536),
               moe=(8, 2, 6144), mixtral=dict(n_head=32, n_kv_head=8, d_ff=4096)),
    # many small experts, a shared one, group-limited choice (no GGUF family has this shape)
    "4k-fine": dict(width=4096, wkv=(64, 64), latent=dict(heads=32, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=1536),
                    moe=(64, 6, 1024), groups=(8, 4), shared=1024, mixtral=None),
}


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


def write_sekolorn(path: str, cfg: dict):
    import torch

    from .safetensors_io import write_safetensors
    os.makedirs(path, exist_ok=True)
    W, d = {}, cfg["width"]
    dev = "cuda" if torch.cuda.is_available() else "cpu"
    g = torch.Generator(device=dev).manual_seed(0)

    def lin(name, *shape):
        W[name] = (torch.randn(*shape, generator=g, device=dev) * shape[-1] ** -0.5).to(torch.bfloat16).cpu()

    def one(name, n):
        W[name] = torch.ones(n, dtype=torch.bfloat16)
    W["embed"] = torch.randn(cfg["vocab"], d, generator=g, device=dev).to(torch.bfloat16).cpu()
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        one(p + "norm1", d)
        one(p + "norm2", d)
        if L["type"] == "wkv":
            HD = m["heads"] * m["dim"]
            for s in "rkvgw":
                W[p + "mix.mu." + s] = torch.full((d,), 0.5, dtype=torch.bfloat16)
            for s in "rkvg":
                lin(p + "mix." + s, HD, d)
            lin(p + "mix.w1", 64, d)
            lin(p + "mix.w2", HD, 64)
            W[p + "mix.w0"] = torch.full((HD,), -3.0, dtype=torch.bfloat16)
            W[p + "mix.u"] = torch.full((m["heads"], m["dim"]), 0.5, dtype=torch.bfloat16)
            one(p + "mix.norm", HD)
            lin(p + "mix.o", d, HD)
        else:
            H, D, RD, VD, R, Q = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank"))
            lin(p + "mix.dq", Q, d)
            one(p + "mix.dq.norm", Q)
            lin(p + "mix.uq", H * (D + RD), Q)
            if "kv_from" not in m:
                lin(p + "mix.dkv", R + RD, d)
                one(p + "mix.dkv.norm", R)
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
    one("final.norm", d)
    lin("head", cfg["vocab"], d)
    with open(os.path.join(path, "config.json"), "w") as fh:
        json.dump(cfg, fh)
    write_safetensors(os.path.join(path, "model.safetensors"), W)


def load(which: str, size: str, model_dir: str, dev):
    from .models.registry import load_model
    sz = SIZES[size]
    os.makedirs(model_dir, exist_ok=True)
    if which == "sekolorn":
        path = os.path.join(model_dir, f"sekolorn-{size}")
        if not os.path.exists(os.path.join(path, "config.json")):
            write_sekolorn(path, sekolorn_config(sz))
    else:
        from .gguf import synth
        # F16 experts run on the dense grouped GEMM's row-major copies (the LDS-dequant GEMM takes K-quants only)
        os.environ.setdefault("NLS_DENSE_WEIGHTS", "1")
        os.environ.setdefault("NLS_DENSE_EXPERTS", "1")
        path = os.path.join(model_dir, f"mixtral-{size}.gguf")
        if not os.path.exists(path):
            name = f"mixtral-{size}"
            synth.SPECS[name] = replace(synth.SPECS["mixtral-8x7b"], name=name, n_layer=4, d_model=sz["width"], vocab=VOCAB,
                                        n_expert=sz["moe"][0], n_expert_used=sz["moe"][1], **sz["mixtral"])
            synth.write_synthetic_gguf(path, name, "F16", seed=0)
    return load_model(path, dev, ctx=None if which != "sekolorn" else 8192)


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
    for size in args.stack_sizes.split(","):
        for which in ("sekolorn", "closest"):
            if args.stack_only not in (None, which) or (which == "closest" and SIZES[size]["mixtral"] is None):
                continue
            t0 = time.time()
            model = load(which, size, args.model_dir, dev)
            t_load = time.time() - t0
            for B, prompt in cases:
                steps = 4 if (B, prompt) in CASES["prefill"] and args.stack != "decode" and not args.stack_case else args.steps
                out = measure(model, B, prompt, min(steps, 100), min(args.warmup, 10))
                print(json.dumps(dict(bench="stack", model=which, size=size, batch=B, prompt=prompt, layers=4,
                                      weights_gb=round(model.weight_bytes / 1e9, 3), load_s=round(t_load, 1),
                                      dtype="bf16" if which == "sekolorn" else "fp16", data="synthetic", **out)), flush=True)
            del model
            torch.cuda.empty_cache()
    return 0
