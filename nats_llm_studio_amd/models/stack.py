"""Decoder stacks assembled from a config: a list of layers, each a mixer plus an optional feed-forward.

A mixer or feed-forward is a class that loads its weights, adds its step buffers, and runs on the rows of a step; a layer
class (OutputNormLayer, SharedNormLayer, SandwichNormLayer) places the norms and joins the sublayers. A looped model runs some layers several
times with the same weights. The per-token cache rows (paged) and the per-sequence states (slots) of all layer runs belong to
the engine, which sees them as `kv_cache` / `state_pool`. Everything runs on the HIP kernels of csrc/stack (ops/stack.py): bf16
operands with an f32 residual, or `dtype=torch.float32` for 32-bit throughout.

Rows of a step are runs of consecutive tokens of one sequence (whole prompts, portions of any size, single decoded
tokens), all in one batch:
  runs     [sequences][4]: first row, rows, state slot, first position   (recurrent layers)
  slot / tok_seq / ctx_len / block_tables                                (paged cache, as in models/llama.py)
"""
from __future__ import annotations

import math
import os
from dataclasses import astuple, dataclass, field
from typing import Dict, List, Optional

import numpy as np
import torch

from ..ops import stack as K
from ..ops import rope_table
from ..safetensors_io import SafetensorsReader
from .llama import ShardSpec
from .stack_config import StackConfig

_SPLIT_WG = 256          # target workgroups of a decode attention launch (one per CU)
_SPLIT_CAP = 64
_SLABS, _SLAB_ROWS = 8, 512      # K splits of an output product, on steps of up to so many rows


@dataclass
class StackBuffers:
    """Device buffers of one step of up to `cap` tokens (static for hipGraph capture). Linear-layer inputs have rows of
    ops.stack.act_ld columns whose padding stays zero."""
    cap: int
    pad: int
    meta: torch.Tensor
    ids: torch.Tensor
    pos: torch.Tensor
    slot: torch.Tensor
    tok_seq: torch.Tensor
    ctx_len: torch.Tensor
    use_prev: torch.Tensor
    block_tables: torch.Tensor
    runs: torch.Tensor
    x: torch.Tensor                     # f32 residual
    xb: Optional[torch.Tensor]          # its bf16 rounding (None: 32-bit model, the residual itself is the operand)
    h: Optional[torch.Tensor]           # normed residual that the sublayers read (None: they read the residual)
    h2: Optional[torch.Tensor]          # with its second norm: what the feed-forward reads (None: the same)
    xx: Optional[torch.Tensor]          # looped models: [x | embedding output], the operand ahead of each pass
    y: Optional[torch.Tensor]           # f32 sublayer output (layers with a shared norm: the slabs of their output product)
    hn: torch.Tensor                    # normed rows of the head
    logits: torch.Tensor
    next_ids: torch.Tensor
    shared: Dict[tuple, torch.Tensor] = field(default_factory=dict)    # scratch shared between layers
    launches: Dict[tuple, object] = field(default_factory=dict)

    @property
    def slab_rows(self) -> int:
        return min(self.pad, _SLAB_ROWS)

    @property
    def act(self) -> torch.Tensor:
        """What the sublayers read."""
        return self.h if self.h is not None else self.x if self.xb is None else self.xb


class _Part:
    """A mixer or feed-forward of layer i: weights `w(name)` are '<layer>.<mix|mlp>.<name>'. Layers that use another's weights
    (weights_of) share its parts: a part keeps nothing of a sequence, its cache and state come with each run."""
    cache_width = 0               # cache elements per token
    plan_bytes = 0                # scratch per context token of a planned prompt run
    plan_run = None               # runs of at least this many tokens take the planned prompt attention (None: never)

    def state_shapes(self) -> Dict[str, int]:
        return {}

    def new_cache(self, slots: int):
        """Cache rows of one layer: [slots, width]."""
        return torch.zeros(slots, self.cache_width, dtype=self.m.dtype, device=self.m.device)

    def __init__(self, model: "StackModel", i: int, cfg, prefix: str):
        self.m, self.i, self.cfg, self.prefix = model, i, cfg, prefix

    def t(self, name: str) -> torch.Tensor:
        return self.m.reader.tensor(self.prefix + name)

    def vec(self, name: str) -> torch.Tensor:
        return self.t(name).to(device=self.m.device, dtype=torch.float32).reshape(-1).contiguous()

    def lin(self, w, shape=None) -> K.PackedLinear:
        w = self.t(w) if isinstance(w, str) else w
        if shape is not None and tuple(w.shape) != tuple(shape):
            raise ValueError(f"{self.prefix}: a weight of shape {tuple(w.shape)}, expected {tuple(shape)}")
        p = K.PackedLinear(w, self.m.f32, self.m.device)
        self.m.weight_bytes += p.nbytes
        return p

    def scratch(self, b: StackBuffers, name: str, rows: int, cols: int, dtype=None) -> torch.Tensor:
        """A zeroed [rows, cols] buffer shared by every layer that asks for this name and shape (same layout: what one
        layer leaves in the padding columns is what the next would)."""
        key = (name, rows, cols, dtype or self.m.dtype)
        if key not in b.shared:
            b.shared[key] = torch.zeros(rows, cols, dtype=dtype or self.m.dtype, device=self.m.device)
        return b.shared[key]


class WkvMixer(_Part):
    """Token-shift mixes -> r | k | v | gate | decay projections -> gated linear recurrence with a per-channel decay
    -> per-head RMS norm, norm weight and gate -> output projection."""
    SHIFTS = ("r", "k", "v", "g", "w")

    def __init__(self, model, i, cfg, prefix):
        super().__init__(model, i, cfg, prefix)
        d, HD = model.cfg.d_model, cfg.heads * cfg.dim
        if cfg.dim > 256:
            raise ValueError(f"wkv head dim {cfg.dim} > 256")
        self.mu = torch.stack([self.vec("mu." + s) for s in self.SHIFTS]).contiguous()
        self.r, self.k, self.v, self.g = (self.lin(n, (HD, d)) for n in ("r", "k", "v", "g"))
        self.w1, self.w2, self.o = self.lin("w1"), self.lin("w2"), self.lin("o", (d, HD))
        self.w0, self.u, self.norm = self.vec("w0"), self.vec("u"), self.vec("norm")

    def state_shapes(self):
        c = self.cfg
        return {"S": c.heads * c.dim * c.dim, "prev": self.m.cfg.d_model}

    def bind(self, b: StackBuffers) -> dict:
        d, HD, P = self.m.cfg.d_model, self.cfg.heads * self.cfg.dim, b.pad
        mix = self.scratch(b, "wkv.mix", len(self.SHIFTS) * P, K.act_ld(d)).view(len(self.SHIFTS), P, -1)
        ld = K.act_ld(HD)
        r, k, v, g, out = (self.scratch(b, "wkv." + n, P, ld) for n in ("r", "k", "v", "g", "out"))
        low = self.scratch(b, "wkv.low", P, K.act_ld(self.w1.N))
        w, o = (self.scratch(b, "wkv." + n, P, ld, torch.float32) for n in ("w", "o"))
        return dict(
            mix=mix, r=r, k=k, v=v, g=g, w=w, o=o, out=out,
            proj=K.LinLaunch([K.Seg(self.r, mix[0], r), K.Seg(self.k, mix[1], k), K.Seg(self.v, mix[2], v),
                              K.Seg(self.g, mix[3], g, "silu"), K.Seg(self.w1, mix[4], low, "tanh")]),
            decay=K.LinLaunch([K.Seg(self.w2, low, w, "decay", bias=self.w0)]),
            o_proj=K.LinLaunch([K.Seg(self.o, out, b.y)]))

    def run(self, b: StackBuffers, e: dict, cache, state, step: "_Step"):
        c, st, T = self.cfg, step.st, step.T
        S, prev = state["S"], state["prev"]
        K.shift_mix(b.x, self.mu, prev, e["mix"], b.runs, b.tok_seq, T, st)
        e["proj"].run(T, st)
        e["decay"].run(T, st)
        if T == step.nruns and c.dim % 4 == 0:          # single tokens only
            K.wkv_step(e["r"], e["k"], e["v"], e["w"], self.u, S, b.x, prev, b.runs, T, self.norm, e["g"], e["out"], c.heads,
                       c.dim, self.m.cfg.eps, st)
            e["o_proj"].run(T, st)
            return
        K.wkv_scan(e["r"], e["k"], e["v"], e["w"], self.u, e["o"], S, b.x, prev, b.runs, step.nruns, c.heads, c.dim, st)
        K.scan_out(e["o"], self.norm, e["g"], e["out"], c.heads, c.dim, T, self.m.cfg.eps, st)
        e["o_proj"].run(T, st)


class LatentMixer(_Part):
    """Latent attention. The cache holds, per token, the normed latent and one rotated key part shared by all heads; a
    layer with kv_from reads an earlier layer's rows. The key up-projection is folded into the query and the value
    up-projection applied to the attended latent, so every head attends over the same cached rows. Long runs (prompt
    chunks) instead expand their context's keys and values once and attend per head (`plan` of the step)."""

    def __init__(self, model, i, cfg, prefix):
        super().__init__(model, i, cfg, prefix)
        c, d = cfg, model.cfg.d_model
        H, D, RD, VD, R, Q = c.heads, c.dim, c.rot_dim, c.vdim, c.kv_rank, c.q_rank
        self.Rp, self.rp = K.latent_pad(R), K.rot_pad(RD)
        self.Dp = self.Rp + self.rp
        self.Dq = K.act_ld(D)                              # unrotated query columns per head
        self.RD4 = K.pad_to(RD, 4)
        self.dq, self.dqn = self.lin("dq", (Q, d)), self.vec("dq.norm")
        self.owner = c.kv_from is None
        if self.owner:
            self.dkv, self.dkvn = self.lin("dkv", (R + RD, d)), self.vec("dkv.norm")
        uq = self.t("uq").to(model.device).view(H, D + RD, Q)
        zero = uq.new_zeros
        self.uqn = self.lin(torch.cat([uq[:, :D], zero(H, self.Dq - D, Q)], 1).reshape(H * self.Dq, Q))
        self.uqr = self.lin(torch.cat([uq[:, D:], zero(H, self.RD4 - RD, Q)], 1).reshape(H * self.RD4, Q))
        # expanded form: per-head keys / values of prompt contexts
        self.xk, self.xr, self.xv = (K.expand_width(*a) for a in (("key", D), ("rot", RD), ("value", VD)))
        self.expand = not model.f32 and None not in (self.xk, self.xr, self.xv)
        if self.expand:
            uk, uv = self.t("uk").to(model.device).view(H, D, R), self.t("uv").to(model.device).view(H, VD, R)
            self.xuk = self.lin(torch.cat([uk, zero(H, self.xk - D, R)], 1).reshape(H * self.xk, R))
            self.xuv = self.lin(torch.cat([uv, zero(H, self.xv - VD, R)], 1).reshape(H * self.xv, R))
        self.uk = self.lin(self.t("uk").to(model.device).view(H, D, R).transpose(1, 2).contiguous())   # [H][R][D]
        self.uv = self.lin(self.t("uv").to(model.device).view(H, VD, R))                               # [H][VD][R]
        self.g, self.o = self.lin("g", (H, d)), self.lin("o", (d, H * VD))
        self.cs = model.rope(c.rot_base, RD)
        self.attends = True
        self.plan_bytes = H * (self.xk + self.xv) * 2 if self.expand else 0

    @property
    def cache_width(self) -> int:
        return self.Dp if self.owner else 0

    @property
    def plan_run(self):
        return _EXPAND_RUN if self.expand else None

    def bind(self, b: StackBuffers) -> dict:
        c, P = self.cfg, b.pad
        H, f = c.heads, torch.float32
        dq = self.scratch(b, "lat.dq", P, c.q_rank, f)
        dkv = self.scratch(b, "lat.dkv", P, c.kv_rank + c.rot_dim, f) if self.owner else None
        gate = self.scratch(b, "lat.gate", P, H, f)
        cq = self.scratch(b, "lat.cq", P, K.act_ld(c.q_rank))
        qn = self.scratch(b, "lat.qn", P, H * self.Dq)
        # (columns between the written parts stay zero: the buffer is shared only between equal layouts)
        q = self.scratch(b, f"lat.q{c.kv_rank}.{c.rot_dim}", P, H * self.Dp)
        lat = self.scratch(b, f"lat.o{c.kv_rank}", P, H * self.Rp)
        ao = self.scratch(b, "lat.ao", P, K.act_ld(H * c.vdim))
        hb = K.latent_head_groups(H, self.Rp)              # workgroups per (token, split)
        n = (_SPLIT_WG // hb + 1) * H
        po = self.scratch(b, "lat.po", 1, n * self.Rp, f)
        pm = self.scratch(b, "lat.pm", 1, n * 2, f)
        down = [K.Seg(self.dq, b.act, dq), K.Seg(self.g, b.act, gate, "sigmoid")]
        if self.owner:
            down.append(K.Seg(self.dkv, b.act, dkv))
        return dict(
            dq=dq, dkv=dkv, cq=cq, q=q, qn=qn, gate=gate, ao=ao, lat=lat, part=(po, pm), hb=hb,
            down=K.LinLaunch(down),
            up=K.LinLaunch([K.Seg(self.uqn, cq, qn),
                            K.Seg(self.uqr, cq, q, "rope", ycol=self.Rp, block=(self.RD4, self.Dp),
                                  rope=(self.cs, b.pos, c.rot_dim // 2))]),
            absorb=K.LinLaunch([K.Seg(self.uk, qn, q, xgs=self.Dq, ygs=self.Dp)]),
            value=K.LinLaunch([K.Seg(self.uv, lat, ao, "gate", xgs=self.Rp, ygs=c.vdim, gate=gate)]),
            o_proj=K.LinLaunch([K.Seg(self.o, ao, b.y)]))

    def run(self, b: StackBuffers, e: dict, cache, state, step: "_Step"):
        c, st, T = self.cfg, step.st, step.T
        rows = cache[step.layer if self.owner else c.kv_from]
        e["down"].run(T, st)
        K.latent_rows(e["dq"], self.dqn, e["cq"], e["dkv"], self.dkvn if self.owner else None, c.kv_rank, self.Rp,
                      c.rot_dim, self.cs, b.pos, b.slot, rows if self.owner else None, T, self.m.cfg.eps, st)
        e["up"].run(T, st)
        plan = step.plan
        if plan is None or plan.rest:
            # latent-space attention of the rows outside the expanded runs (the others have no keys here)
            e["absorb"].run(T, st)
            ns = 1 if self.m.f32 else max(1, min(_SPLIT_CAP, _SPLIT_WG // (T * e["hb"])))
            K.latent_attention(e["q"], rows, e["lat"], e["part"], b.block_tables, step.block_size, b.tok_seq,
                               b.ctx_len if plan is None else plan.actx, T, c.heads, ns, self.Rp, self.rp, c.scale, st)
            e["value"].run(T, st)
        if plan is not None:
            kx, vx, lin = self._expansion(b, e, rows, plan)
            lin.run(plan.nx, st)
            K.latent_prefill(e["qn"], self.Dq, e["q"], self.Rp, self.Dp, kx, vx, rows, plan.xmap, plan.blocks, plan.nblocks,
                             plan.waves, e["gate"], e["ao"], c.heads, self.xk, self.xr, self.xv, c.vdim, c.scale, st)
        e["o_proj"].run(T, st)

    def _expansion(self, b: StackBuffers, e: dict, rows, plan):
        """Scratch for the expanded keys / values (shared by the layers, grown on demand) and the launch that fills it."""
        H = self.cfg.heads
        kx = self.m.grown(b, "lat.kx", plan.nx, H * self.xk)
        vx = self.m.grown(b, "lat.vx", plan.nx, H * self.xv)
        key = (kx.data_ptr(), vx.data_ptr(), rows.data_ptr(), plan.xmap.data_ptr())
        if e.get("expand_key") != key:
            e["expand_key"] = key
            e["expand"] = K.LinLaunch([K.Seg(self.xuk, rows, kx, xmap=plan.xmap), K.Seg(self.xuv, rows, vx, xmap=plan.xmap)])
        return kx, vx, e["expand"]


class MoeFeedForward(_Part):
    """Routed experts (two matrices with a squared relu, or three with a silu gate) chosen by group-limited scores, plus a shared
    expert. Leaves the experts' output rows in `ye`; the caller's output norm combines them."""
    EPI = {"relu2": "relu2", "silu_glu": "siluglu"}

    def __init__(self, model, i, cfg, prefix):
        super().__init__(model, i, cfg, prefix)
        d, E = model.cfg.d_model, cfg.experts
        self.router = self.lin("router", (E, d))
        self.glu = model.cfg.design.expert_act == "silu_glu"
        self.up = self.lin(torch.stack([self.first(f"e{j}.") for j in range(E)]), (E, cfg.ff * (1 + self.glu), d))
        self.down = self.lin(torch.stack([self.t(f"e{j}.down") for j in range(E)]), (E, d, cfg.ff))
        if cfg.shared_ff:
            self.sup = self.lin(self.first("shared."), (cfg.shared_ff * (1 + self.glu), d))
            self.sdown = self.lin("shared.down", (d, cfg.shared_ff))

    def first(self, name: str) -> torch.Tensor:
        """The matrix ahead of the activation; gate and up rows alternate."""
        up = self.t(name + "up")
        return torch.stack([self.t(name + "gate"), up], 1).reshape(-1, up.shape[1]) if self.glu else up

    def bind(self, b: StackBuffers) -> dict:
        c, P = self.cfg, b.pad
        k = c.top
        design = self.m.cfg.design
        act = self.EPI[design.expert_act]
        key = ("plan", c.experts, k, c.groups, c.keep, c.scale)
        plan = b.launches.get(key)
        if plan is None:
            plan = b.launches[key] = K.MoePlan(P, c.experts, k, c.groups, c.keep, c.scale, self.m.device, design.router_score,
                                               {"top2": 2, "max": 1}[design.router_group])
        z = self.scratch(b, "moe.z", P, c.experts, torch.float32)
        h = self.scratch(b, "moe.h", P * k, K.act_ld(c.ff))
        ye = self.scratch(b, "moe.y", P * (k + 1), self.m.cfg.d_model, torch.float32)
        first = [K.Seg(self.router, b.act, z)]
        down = [K.Seg(self.down, h, ye, routed=(plan.rows, 1))]
        if c.shared_ff:
            hs = self.scratch(b, "moe.hs", P, K.act_ld(c.shared_ff))
            first.append(K.Seg(self.sup, b.act, hs, act))
            down.append(K.Seg(self.sdown, hs, ye, yrow=P * k))
        return dict(plan=plan, z=z, ye=ye, first=K.LinLaunch(first), shared_row0=P * k if c.shared_ff else -1,
                    up=K.LinLaunch([K.Seg(self.up, b.act, h, act, routed=(plan.rows, k))], plan),
                    down=K.LinLaunch(down, plan))

    def run(self, b: StackBuffers, e: dict, step: "_Step"):
        T, st = step.T, step.st
        e["first"].run(T, st)
        e["plan"].run(e["z"], T, st)
        e["up"].run(T, st)
        e["down"].run(T, st)


class _SharedPart(_Part):
    """A part of a SharedNormLayer (or of a SandwichNormLayer, which has one in each half): reads the layer's normed input through segments of the layer's one input launch and leaves
    its operand of the layer's one output product in `out` (columns of a shared buffer). `scale` weights its output; it goes
    into a 32-bit factor that the operand is multiplied with anyway, so it costs no rounding."""
    out_width = 0                 # columns of the operand, a multiple of 64

    def __init__(self, model, i, cfg, prefix, scale: float = 1.0):
        super().__init__(model, i, cfg, prefix)
        self.scale = scale

    def mat(self, name: str, shape) -> torch.Tensor:
        w = self.t(name)
        if tuple(w.shape) != tuple(shape):
            raise ValueError(f"{self.prefix}{name}: a weight of shape {tuple(w.shape)}, expected {tuple(shape)}")
        return w.to(self.m.device)

    def vecn(self, name: str, n: int) -> torch.Tensor:
        v = self.vec(name)
        if v.numel() != n:
            raise ValueError(f"{self.prefix}{name}: {v.numel()} values, expected {n}")
        return v

    def out_weight(self) -> torch.Tensor:
        """[width of the model, out_width]: the output projection, zero in the operand's padding columns."""
        raise NotImplementedError

    def bind(self, b: StackBuffers, out: torch.Tensor, x: torch.Tensor) -> dict:
        """Step buffers and launches; "inputs": the segments of the layer's input launch, which read x."""
        raise NotImplementedError


class AttentionPart(_SharedPart):
    """Grouped-query softmax attention: queries and keys optionally RMS-normed over their whole projections or (rotated) per
    head, rotary positions on the first columns of each head, values projected on their own or equal to the projected keys,
    optionally a sigmoid gate per head or per output column, a sliding window with kept first keys, one more in the denominator,
    heads whose softmax weights are mixed. The cache holds the finished keys and the values, [2][slots][kv_heads * padded head]."""

    def __init__(self, model, i, cfg, prefix, scale=1.0):
        super().__init__(model, i, cfg, prefix, scale)
        c, d, design = cfg, model.cfg.d_model, model.cfg.design
        H, G, D, V = c.heads, c.kv_heads, c.dim, c.vdim
        self.attends = True
        self.Dp, self.mfma = K.head_pad(max(D, V))
        self.mfma = self.mfma and not model.f32
        self.own_values = design.attn_values == "projection"
        names = [("q", H * D), ("k", G * D)] + ([("v", G * V)] if self.own_values else [])
        w = {n: self.mat(n, (rows, d)) for n, rows in names}
        if design.rotary == "halves":
            # columns i and i + dims / 2 of a head become neighbours: scores and norms do not see the order
            half = torch.arange(c.rot_dims, device=model.device).view(2, -1).T.reshape(-1)
            order = torch.cat([half, torch.arange(c.rot_dims, D, device=model.device)])
            for n, heads in (("q", H), ("k", G)):
                w[n] = w[n].view(heads, D, d)[:, order].reshape(heads * D, d)
        self.qkv = self.lin(torch.cat([w[n] for n, _ in names]))
        self.mask = dict(window=c.window, keep=c.keep_first, sink=design.attn_sink)
        if design.attn_gate != "head" and scale != 1.0:
            raise ValueError("a weighted attention output needs its head gate")
        if (design.attn_gate == "column") != design.attn_talk:
            raise NotImplementedError("a gate per column and mixed heads come together")
        self.qn = self.kn = None
        if design.attn_qk_norm == "projection":
            self.qn, self.kn = self.vecn("q.norm", H * D), self.vecn("k.norm", G * D)
        self.g = self.lin("g", (H if design.attn_gate == "head" else H * V, d)) if design.attn_gate else None
        self.cs = model.rope(c.rot_base, c.rot_dims, c.rot_scaling) if c.rot_dims else None
        self.talk = None
        if design.attn_talk:
            self.talk_plan = K.TalkPlan(H, G, self.Dp, c.window, model.cfg.ctx, model.f32, model.device, c.scale)
            self.talk = self.talk_plan.matrix(self.mat("talk", (H, H)))
        self.cache_width = 2 * G * self.Dp
        self.out_width = K.act_ld(H * self.Dp)
        self.groups = K.attn_groups(H, G)

    @property
    def plan_run(self):
        return _FLASH_RUN if (self.mfma if self.talk is None else self.talk_plan.prefill) else None

    def new_cache(self, slots):
        return torch.zeros(2, K.pad_to(slots, K.KEY_TILE), self.cfg.kv_heads * self.Dp, dtype=self.m.dtype, device=self.m.device)

    def out_weight(self):
        c, d = self.cfg, self.m.cfg.d_model
        w = self.mat("o", (d, c.heads * c.vdim)).view(d, c.heads, c.vdim)
        w = torch.nn.functional.pad(w, (0, self.Dp - c.vdim)).reshape(d, c.heads * self.Dp)
        return torch.nn.functional.pad(w, (0, self.out_width - w.shape[1]))

    def bind(self, b, out, x):
        c, P, f = self.cfg, b.pad, torch.float32
        H, G, D = c.heads, c.kv_heads, c.dim
        qkv = self.scratch(b, "attn.qkv", P, K.pad_to(self.qkv.N, 4), f)
        gate = None
        if self.g is not None:                            # per column: in the activation type, 16-byte rows
            gate = self.scratch(b, "attn.gate", P, H, f) if self.talk is None else \
                self.scratch(b, "attn.cgate", P, K.pad_to(self.g.N, 8))
        q = self.scratch(b, f"attn.q{D}", P, H * self.Dp)
        k0 = H * D
        e = dict(q=q, gate=gate, out=out, qp=qkv, kp=qkv[:, k0:], vp=qkv[:, k0 + G * D:] if self.own_values else qkv[:, k0:],
                 inputs=[K.Seg(self.qkv, x, qkv)] + ([K.Seg(self.g, x, gate, "sigmoid", alpha=self.scale)]
                                                     if self.g is not None else []))
        if self.talk is not None:
            if self.talk_plan.mfma:
                sizes = self.talk_plan.scratch(P)
                names = ("talk.sc", "talk.st", "talk.po", "talk.cnt")
                e["part"] = [self.scratch(b, n, 1, s, f if n != "talk.cnt" else torch.int32) for n, s in zip(names, sizes)]
                e["part"] = [t.view(-1) for t in e["part"]]
            return e
        n = _SPLIT_WG // self.groups + 1                  # rows x splits
        e["part"] = (self.scratch(b, "attn.po", 1, n * H * self.Dp, f), self.scratch(b, "attn.pm", 1, n * H * 2, f),
                     self.scratch(b, "attn.cnt", 1, _SPLIT_WG + self.groups, torch.int32))
        return e

    def run(self, b, e, cache, state, step: "_Step"):
        c, st, T = self.cfg, step.st, step.T
        kc, vc = cache[0], cache[1]
        K.attn_rows(e["qp"], e["kp"], e["vp"], self.qn, self.kn, self.cs, b.pos, b.slot, e["q"], kc, vc, T, c.heads,
                    c.kv_heads, c.dim, self.Dp, c.rot_dims, self.m.cfg.eps, st, V=c.vdim,
                    head_norm=self.m.cfg.design.attn_qk_norm == "head", key_tiles=self.talk is not None and self.talk_plan.mfma)
        plan = step.plan
        if self.talk is not None:
            args = (self.talk_plan, e["q"], kc, vc, self.talk, e["gate"], e["out"])
            if plan is None or plan.rest:
                K.talk_attention(*args, e.get("part"), b.block_tables, step.block_size, b.tok_seq,
                                 b.ctx_len if plan is None else plan.actx, T, c.vdim, c.scale, st)
            if plan is not None:
                K.talk_prefill(*args, b.block_tables, step.block_size, plan.blocks, plan.nblocks, plan.waves, c.vdim, c.scale, st)
            return
        if plan is None or plan.rest:
            ns = max(1, min(_SPLIT_CAP, _SPLIT_WG // (T * self.groups))) if self.mfma else 1
            K.gqa_attention(e["q"], kc, vc, e["gate"], e["out"], e["part"], b.block_tables, step.block_size, b.tok_seq,
                            b.ctx_len if plan is None else plan.actx, T, c.heads, c.kv_heads, self.Dp, self.mfma, ns,
                            c.scale, st, **self.mask)
        if plan is not None:
            K.gqa_prefill(e["q"], kc, vc, plan.xmap, plan.blocks, plan.nblocks, plan.waves, e["gate"], e["out"], c.heads,
                          c.kv_heads, self.Dp, c.scale, st, **self.mask)


class GlaPart(_SharedPart):
    """Gated linear attention: a recurrent state per head, decayed per key channel by a low-rank gate, read after each
    token's update; per-head RMS norm, one weight for all heads, silu gate."""

    def __init__(self, model, i, cfg, prefix, scale=1.0):
        super().__init__(model, i, cfg, prefix, scale)
        c, d = cfg, model.cfg.d_model
        H, D, V = c.heads, c.dim, c.vdim
        if D > 256:
            raise ValueError(f"gated linear attention: key width {D} > 256")
        a1 = self.t("a1").to(model.device)
        # one buffer [q | k | v | zeros | a1]: the low-rank gate input starts at a linear layer's alignment
        self.low = K.act_ld(H * (2 * D + V))
        qkv = torch.cat([self.mat("q", (H * D, d)), self.mat("k", (H * D, d)), self.mat("v", (H * V, d))])
        self.qkva = self.lin(torch.cat([qkv, qkv.new_zeros(self.low - qkv.shape[0], d), a1]))
        self.ld = self.low + K.act_ld(a1.shape[0])
        self.a2, self.a2b = self.lin("a2", (H * D, a1.shape[0])), self.vecn("a2.b", H * D)
        # decode steps make the decays themselves (a row-major copy of a2) unless the rank is large
        self.a2r = self.t("a2").to(device=model.device, dtype=model.dtype).contiguous() if a1.shape[0] <= 64 else None
        self.g = self.lin("g", (H * V, d))
        self.norm = (self.vecn("norm", V) * scale).repeat(H).contiguous()
        self.out_width = K.act_ld(H * V)

    def state_shapes(self):
        c = self.cfg
        return {"S": c.heads * c.dim * c.vdim}

    def out_weight(self):
        c, d = self.cfg, self.m.cfg.d_model
        return torch.nn.functional.pad(self.mat("o", (d, c.heads * c.vdim)), (0, self.out_width - c.heads * c.vdim))

    def bind(self, b, out, x):
        c, P, f = self.cfg, b.pad, torch.float32
        HD, HV = c.heads * c.dim, c.heads * c.vdim
        z = self.scratch(b, "gla.qkva", P, self.ld)
        a = self.scratch(b, "gla.a", P, HD, f)
        o = self.scratch(b, "gla.o", P, HV, f) if c.vdim > 128 else None
        g = self.scratch(b, "gla.g", P, HV)
        return dict(q=z, k=z[:, HD:], v=z[:, 2 * HD:], low=z[:, self.low:], a=a, o=o, g=g, out=out,
                    inputs=[K.Seg(self.qkva, x, z), K.Seg(self.g, x, g, "silu")],
                    decay=K.LinLaunch([K.Seg(self.a2, z, a, "sigpow", xcol=self.low, bias=self.a2b, alpha=1.0 / c.tau)]))

    def run(self, b, e, cache, state, step: "_Step"):
        c, st, T, eps = self.cfg, step.st, step.T, self.m.cfg.eps
        H, D, V, S, qs = c.heads, c.dim, c.vdim, state["S"], c.dim ** -0.5
        single = T == step.nruns and V % 4 == 0 and V <= 1024
        a = None if single and self.a2r is not None else e["a"]
        if a is not None:
            e["decay"].run(T, st)
        if single:
            K.gla_step(e["q"], e["k"], e["v"], a, (e["low"], self.a2r, self.a2b, 1.0 / c.tau), qs, S, b.runs, T, self.norm,
                       e["g"], e["out"], H, D, V, eps, st)
            return
        n = step.nruns
        shape = K.gla_shape(T, n, H, V)
        seg = None
        if shape[0] > 1:
            seg = (self.m.grown(b, "gla.seg", n * shape[0], H * D * V, torch.float32),
                   self.m.grown(b, "gla.segw", n * shape[0], H * D, torch.float32))
        fused = V <= 64 * shape[1]
        K.gla_scan(e["q"], e["k"], e["v"], e["a"], qs, e["o"], self.norm, e["g"], e["out"] if fused else None, S, b.runs, n, H, D,
                   V, eps, shape, seg, st)
        if not fused:
            K.scan_out(e["o"], self.norm, e["g"], e["out"], H, V, T, eps, st)


class LightningPart(_SharedPart):
    """Linear attention with one constant decay per head: silu on queries, keys and values, a recurrent state per head read
    after each token's update; RMS norm over all heads' outputs together, sigmoid gate. Runs on the kernels of gated linear
    attention, whose decays are a row that every token shares."""

    def __init__(self, model, i, cfg, prefix, scale=1.0):
        super().__init__(model, i, cfg, prefix, scale)
        c, d = cfg, model.cfg.d_model
        H, D, V = c.heads, c.dim, c.vdim
        if D > 256 or H * V > 16384:
            raise ValueError(f"lightning attention: key width {D} > 256 or {H} x {V} outputs > 16384")
        self.qkv = self.lin(torch.cat([self.mat("q", (H * D, d)), self.mat("k", (H * D, d)), self.mat("v", (H * V, d))]))
        self.g = self.lin("g", (H * V, d))
        self.norm = (self.vecn("norm", H * V) * scale).contiguous()
        self.a = torch.tensor(c.decay, dtype=torch.float32, device=model.device).repeat_interleave(D)[None].expand(2, -1)
        self.out_width = K.act_ld(H * V)

    def state_shapes(self):
        c = self.cfg
        return {"S": c.heads * c.dim * c.vdim}

    def out_weight(self):
        c, d = self.cfg, self.m.cfg.d_model
        return torch.nn.functional.pad(self.mat("o", (d, c.heads * c.vdim)), (0, self.out_width - c.heads * c.vdim))

    def bind(self, b, out, x):
        c, P = self.cfg, b.pad
        HD, HV = c.heads * c.dim, c.heads * c.vdim
        z = self.scratch(b, "lightning.qkv", P, K.pad_to(2 * HD + HV, 8))
        o = self.scratch(b, "lightning.o", P, K.pad_to(HV, 4), torch.float32)
        g = self.scratch(b, "lightning.g", P, K.pad_to(HV, 8))
        return dict(q=z, k=z[:, HD:], v=z[:, 2 * HD:], o=o, g=g, out=out,
                    inputs=[K.Seg(self.qkv, x, z, "silu"), K.Seg(self.g, x, g, "sigmoid")])

    def run(self, b, e, cache, state, step: "_Step"):
        c, st, T, n, eps = self.cfg, step.st, step.T, step.nruns, self.m.cfg.eps
        H, D, V, S = c.heads, c.dim, c.vdim, state["S"]
        if T == n and V % 4 == 0 and V <= 1024:
            K.gla_step(e["q"], e["k"], e["v"], self.a, None, 1.0, S, b.runs, T, None, None, None, H, D, V, eps, st, o=e["o"])
        else:
            shape = K.gla_shape(T, n, H, V)
            seg = None
            if shape[0] > 1:
                seg = (self.m.grown(b, "gla.seg", n * shape[0], H * D * V, torch.float32),
                       self.m.grown(b, "gla.segw", n * shape[0], H * D, torch.float32))
            K.gla_scan(e["q"], e["k"], e["v"], self.a, 1.0, e["o"], None, None, None, S, b.runs, n, H, D, V, eps, shape, seg, st)
        K.row_norm(e["o"], None, self.norm, e["out"], T, eps, st, rms=True, gate=e["g"])


class DeltaPart(_SharedPart):
    """Gated delta rule: queries, keys and values through a short causal convolution and silu, unit queries and keys, a recurrent
    state per head with a low-rank decay per key channel, corrected by each token towards its value; per-head RMS norm, one
    weight for all heads, a low-rank sigmoid gate."""

    def __init__(self, model, i, cfg, prefix, scale=1.0):
        super().__init__(model, i, cfg, prefix, scale)
        c, d, dev = cfg, model.cfg.d_model, model.device
        H, G, D, V = c.heads, c.kv_heads, c.dim, c.vdim
        if D > 256:
            raise ValueError(f"delta rule: key width {D} > 256")
        a1, g1 = self.t("a1").to(dev), self.t("g1").to(dev)
        self.ra, self.rg = a1.shape[0], g1.shape[0]
        # one buffer [q | k | v | zeros | a1 | zeros | g1]: the low-rank inputs start at a linear layer's alignment
        self.nch = 2 * G * D + H * V
        self.low, qkv = K.act_ld(self.nch), [self.mat("q", (G * D, d)), self.mat("k", (G * D, d)), self.mat("v", (H * V, d))]
        self.lowg = self.low + K.act_ld(self.ra)
        gap = lambda n: a1.new_zeros(n, d)      # noqa: E731
        self.zw = self.lin(torch.cat(qkv + [gap(self.low - self.nch), a1, gap(self.lowg - self.low - self.ra), g1]))
        self.ld = self.lowg + K.act_ld(self.rg)
        self.conv = torch.cat([self.mat(n + ".conv", (w, c.conv)) for n, w in (("q", G * D), ("k", G * D), ("v", H * V))])
        self.conv = self.conv.to(torch.float32).contiguous()
        self.b = self.lin("b", (H, d))
        # exp(-A softplus(z)) = sigmoid(-z)^A
        a2, g2 = -self.mat("a2", (H * D, self.ra)), self.mat("g2", (H * V, self.rg))
        self.a2, self.g2 = self.lin(a2), self.lin(g2)
        self.a2r, self.g2r = (w.to(model.dtype).contiguous() for w in (a2, g2))
        self.dt = -self.vecn("dt_bias", H * D)
        self.rate = self.vecn("A_log", H).exp().repeat_interleave(D).contiguous()
        self.norm = (self.vecn("norm", V) * scale).repeat(H).contiguous()
        self.out_width = K.act_ld(H * V)

    def state_shapes(self):
        c = self.cfg
        s = {"S": c.heads * c.dim * c.vdim}
        if c.conv > 1:
            s["conv"] = (c.conv - 1) * self.nch
        return s

    def out_weight(self):
        c, d = self.cfg, self.m.cfg.d_model
        return torch.nn.functional.pad(self.mat("o", (d, c.heads * c.vdim)), (0, self.out_width - c.heads * c.vdim))

    def bind(self, b, out, x):
        c, P, f = self.cfg, b.pad, torch.float32
        HD, HV, GD = c.heads * c.dim, c.heads * c.vdim, c.kv_heads * c.dim
        z, y = self.scratch(b, "delta.z", P, self.ld), self.scratch(b, "delta.y", P, K.pad_to(self.nch, 8))
        fac, beta = self.scratch(b, "delta.fac", P, 2 * c.kv_heads, f), self.scratch(b, "delta.beta", P, c.heads, f)
        a, g = self.scratch(b, "delta.a", P, HD, f), self.scratch(b, "delta.g", P, K.pad_to(HV, 8))
        o = self.scratch(b, "delta.o", P, HV, f) if c.vdim > 128 else None
        return dict(z=z, q=y, k=y[:, GD:], v=y[:, 2 * GD:], fac=fac, beta=beta, a=a, g=g, o=o, out=out,
                    low=z[:, self.low:], lowg=z[:, self.lowg:],
                    inputs=[K.Seg(self.zw, x, z), K.Seg(self.b, x, beta, "sigmoid")],
                    gates=K.LinLaunch([K.Seg(self.a2, z, a, "sigpow", xcol=self.low, bias=self.dt, gate=self.rate),
                                       K.Seg(self.g2, z, g, "sigmoid", xcol=self.lowg)]))

    def run(self, b, e, cache, state, step: "_Step"):
        c, st, T, n, eps = self.cfg, step.st, step.T, step.nruns, self.m.cfg.eps
        H, G, D, V, S = c.heads, c.kv_heads, c.dim, c.vdim, state["S"]
        single = T == n and V % 4 == 0 and V <= 1024
        rank = max(self.ra, self.rg)
        own = single and (rank <= 64 or (T <= 16 and rank <= 256))    # the step makes its decays and gate itself
        if not own:
            e["gates"].run(T, st)
        K.delta_conv(e["z"], self.conv, e["q"], e["fac"], state.get("conv"), b.runs, b.tok_seq, T, n, H, G, D, V, st)
        qkv = (e["q"], e["k"], e["v"], e["fac"], e["beta"])
        if single:
            K.delta_step(*qkv, None if own else e["a"], (e["low"], self.a2r, self.dt, self.rate), None if own else e["g"],
                         (e["lowg"], self.g2r), self.ld, S, b.runs, T, self.norm, e["out"], H, G, D, V, eps, st)
            return
        shape = K.delta_shape(T, n, H, D, V)
        seg = None
        if shape[0] > 1:
            seg = (self.m.grown(b, "delta.seg", n * shape[0], H * D * V, torch.float32),
                   self.m.grown(b, "delta.segm", n * shape[0], H * D * D, torch.float32))
        fused = V <= 64 * shape[1]
        K.delta_scan(*qkv, e["a"], e["o"], self.norm, e["g"], e["out"] if fused else None, S, b.runs, n, H, G, D, V, eps, shape, seg,
                     st)
        if not fused:
            K.scan_out(e["o"], self.norm, e["g"], e["out"], H, V, T, eps, st)


class DensePart(_SharedPart):
    """Gated dense feed-forward: down(act(gate h) * (up h)), the activation and product in the input launch's epilogue."""
    EPI = {"gelu_tanh": "geglu", "clamped_swiglu": "swiglu"}

    def __init__(self, model, i, cfg, prefix, scale=1.0):
        super().__init__(model, i, cfg, prefix, scale)
        d = model.cfg.d_model
        if scale != 1.0:
            raise ValueError("the feed-forward's output is not weighted")
        gate, up = self.mat("gate", (cfg.ff, d)), self.mat("up", (cfg.ff, d))
        self.gu = self.lin(torch.stack([gate, up], 1).reshape(2 * cfg.ff, d))        # rows alternate
        self.out_width = K.act_ld(cfg.ff)

    def out_weight(self):
        ff = self.cfg.ff
        return torch.nn.functional.pad(self.mat("down", (self.m.cfg.d_model, ff)), (0, self.out_width - ff))

    def bind(self, b, out, x):
        return dict(inputs=[K.Seg(self.gu, x, out, self.EPI[self.m.cfg.design.glu_act], alpha=self.cfg.limit)])

    def run(self, b, e, cache, state, step):
        pass


class PolyNormPart(_SharedPart):
    """Dense feed-forward without a gate: down(a n(z) + b n(z^2) + c n(z^3) + e), z = up h, n an RMS norm over the token's values."""

    def __init__(self, model, i, cfg, prefix, scale=1.0):
        super().__init__(model, i, cfg, prefix, scale)
        self.up = self.lin(self.mat("up", (cfg.ff, model.cfg.d_model)))
        self.act = self.vecn("act", 4)
        self.out_width = K.act_ld(cfg.ff)

    def out_weight(self):
        ff = self.cfg.ff
        return torch.nn.functional.pad(self.mat("down", (self.m.cfg.d_model, ff)), (0, self.out_width - ff))

    def bind(self, b, out, x):
        z = self.scratch(b, "poly.z", b.pad, K.pad_to(self.cfg.ff, 8))
        return dict(z=z, out=out, inputs=[K.Seg(self.up, x, z)])

    def run(self, b, e, cache, state, step):
        K.poly_norm(e["z"], self.act, e["out"], self.cfg.ff, step.T, self.m.cfg.eps, step.st)


def dense_part(model, i, cfg, prefix, scale=1.0):
    part = PolyNormPart if model.cfg.design.glu_act == "poly_norm" else DensePart
    return part(model, i, cfg, prefix, scale)


class OutputNormLayer:
    """x <- x + norm1(mixer(x)), then x <- x + norm2(feed-forward(x))."""

    def __init__(self, model: "StackModel", i: int, L):
        p = f"l{i}."
        self.m = model
        self.mix = MIXERS[L.mixer.kind](model, i, L.mixer, p + "mix.")
        self.mlp = FEED_FORWARDS[L.mlp.kind](model, i, L.mlp, p + "mlp.") if L.mlp is not None else None
        self.norm1 = model.norm_weight(p + "norm1")
        self.norm2 = model.norm_weight(p + "norm2") if self.mlp is not None else None
        self.parts = [self.mix]

    def bind(self, b: StackBuffers, key):
        b.launches[key, "mix"] = self.mix.bind(b)
        if self.mlp is not None:
            b.launches[key, "mlp"] = self.mlp.bind(b)

    def new_caches(self, slots):
        return self.mix.new_cache(slots) if self.mix.cache_width else None

    def run(self, b, key, kc, state, step: "_Step", fin: dict):
        cfg, st, T = self.m.cfg, step.st, step.T
        rms = cfg.design.norm == "rms"
        self.mix.run(b, b.launches[key, "mix"], kc, state, step)
        K.norm_add(b.y, self.norm1, b.x, b.xb, T, cfg.eps, st, rms=rms, **(fin if self.mlp is None else {}))
        if self.mlp is not None:
            e = b.launches[key, "mlp"]
            self.mlp.run(b, e, step)
            K.norm_add(e["ye"], self.norm2, b.x, b.xb, T, cfg.eps, st, plan=e["plan"], shared_row0=e["shared_row0"], rms=rms,
                       **fin)


class SharedNormLayer:
    """h = norm1(x), x <- x + the sum of the sublayers' outputs on h; or (norm_place "parallel") the feed-forward reads norm2(x).
    The sublayers' input projections are one launch (of up to ops.stack.SEGS segments), their output projections one product
    over the columns of all their operands; the residual add and the next layer's norms are one launch."""

    def __init__(self, model: "StackModel", i: int, L):
        p = f"l{i}."
        self.m = model
        self.norm1 = model.norm_weight(p + "norm1")
        self.parts = [PARTS[c.kind](model, i, c, p + "mix." + sub, scale) for c, sub, scale in mixer_parts(L.mixer)]
        self.norm2 = None
        self.mixers = len(self.parts)
        if L.mlp is not None:
            self.parts.append(PARTS[L.mlp.kind](model, i, L.mlp, p + "mlp."))
            if model.cfg.design.norm_place == "parallel":
                self.norm2 = model.norm_weight(p + "norm2")
        self.o = K.PackedLinear(torch.cat([q.out_weight() for q in self.parts], 1), model.f32, model.device)
        model.weight_bytes += self.o.nbytes

    def bind(self, b: StackBuffers, key):
        widths = [q.out_width for q in self.parts]
        cat = b.shared.get(("cat", sum(widths)))
        if cat is None:
            cat = b.shared["cat", sum(widths)] = torch.zeros(b.pad, sum(widths), dtype=self.m.dtype, device=self.m.device)
        e, c0, segs = [], 0, []
        for j, (q, w) in enumerate(zip(self.parts, widths)):
            e.append(q.bind(b, cat[:, c0:c0 + w], b.h2 if self.norm2 is not None and j >= self.mixers else b.act))
            segs += e[-1]["inputs"]
            c0 += w
        b.launches[key, "parts"] = e
        b.launches[key, "in"] = [K.LinLaunch(segs[o:o + K.SEGS]) for o in range(0, len(segs), K.SEGS)]
        # small steps may split K: slabs of up to 512 rows, added by the residual's launch
        b.launches[key, "out"] = K.LinLaunch([K.Seg(self.o, cat, self.m.slabs(b), slabs=_SLABS, slab_rows=b.slab_rows)])

    def new_caches(self, slots):
        return {j: q.new_cache(slots) for j, q in enumerate(self.parts) if q.cache_width} or None

    def run(self, b, key, kc, state, step: "_Step", fin: dict):
        cfg = self.m.cfg
        for launch in b.launches[key, "in"]:
            launch.run(step.T, step.st)
        caches = kc.get(step.layer, {})
        for j, (q, e) in enumerate(zip(self.parts, b.launches[key, "parts"])):
            q.run(b, e, caches.get(j), state, step)
        n = b.launches[key, "out"].run(step.T, step.st)
        K.norm_add(self.m.slabs(b), None, b.x, fin.pop("copy", None), step.T, cfg.eps, step.st, rms=cfg.design.norm == "rms",
                   slabs=n, slab_rows=b.slab_rows, **fin)


class SandwichNormLayer:
    """x <- x + norm1b(mixer(norm1(x))), then x <- x + norm2b(feed-forward(norm2(x))). The launch that adds a sublayer's output
    (a product's slabs, or routed experts' rows) norms it, and the new residual for what comes next."""

    def __init__(self, model: "StackModel", i: int, L):
        p = f"l{i}."
        self.m = model
        if L.mixer.kind == "parallel":
            raise NotImplementedError("mixers side by side between two norms")
        self.parts = [PARTS[L.mixer.kind](model, i, L.mixer, p + "mix.")]
        self.norm1, self.after = model.norm_weight(p + "norm1"), [model.norm_weight(p + "norm1b")]
        self.norm_ff = None
        if L.mlp is not None:
            part = MoeFeedForward if L.mlp.kind == "moe" else PARTS[L.mlp.kind]
            self.parts.append(part(model, i, L.mlp, p + "mlp."))
            self.norm_ff = model.norm_weight(p + "norm2")
            self.after.append(model.norm_weight(p + "norm2b"))
        self.routed = [isinstance(q, MoeFeedForward) for q in self.parts]
        self.o = [None if r else q.lin(q.out_weight()) for q, r in zip(self.parts, self.routed)]

    def bind(self, b: StackBuffers, key):
        halves = []
        for q, routed, o in zip(self.parts, self.routed, self.o):
            if routed:
                halves.append((q.bind(b), None, None))
                continue
            x = q.scratch(b, "sandwich.out", b.pad, q.out_width)
            e = q.bind(b, x, b.act)
            halves.append((e, [K.LinLaunch(e["inputs"][j:j + K.SEGS]) for j in range(0, len(e["inputs"]), K.SEGS)],
                           K.LinLaunch([K.Seg(o, x, self.m.slabs(b), slabs=_SLABS, slab_rows=b.slab_rows)])))
        b.launches[key, "halves"] = halves

    def new_caches(self, slots):
        q = self.parts[0]
        return q.new_cache(slots) if q.cache_width else None

    def run(self, b, key, kc, state, step: "_Step", fin: dict):
        cfg, T, st = self.m.cfg, step.T, step.st
        for j, (q, (e, inputs, out)) in enumerate(zip(self.parts, b.launches[key, "halves"])):
            if inputs is None:
                q.run(b, e, step)
                y = dict(y=e["ye"], plan=e["plan"], shared_row0=e["shared_row0"])
            else:
                for launch in inputs:
                    launch.run(T, st)
                q.run(b, e, kc.get(step.layer), state, step)
                y = dict(y=self.m.slabs(b), slabs=out.run(T, st), slab_rows=b.slab_rows)
            nxt = fin if j == len(self.parts) - 1 else dict(out_norm=self.norm_ff, out=b.h)
            K.norm_add(w=self.after[j], x=b.x, xb=None, T=T, eps=cfg.eps, st=st, rms=cfg.design.norm == "rms", groups=cfg.norm_groups,
                       **y, **nxt)


def mixer_parts(c) -> list:
    """The parts of a mixer on a shared normed input: (config, tensor prefix, weight of the output)."""
    if c.kind == "parallel":
        return [(c.left, "left.", c.left_scale), (c.right, "right.", c.right_scale)]
    return [(c, "", 1.0)]


MIXERS = {"wkv": WkvMixer, "latent_attention": LatentMixer}
FEED_FORWARDS = {"moe": MoeFeedForward}
PARTS = {"attention": AttentionPart, "gla": GlaPart, "lightning": LightningPart, "channel_delta": DeltaPart,
         "dense": dense_part}
LAYERS = {"output": OutputNormLayer, "shared": SharedNormLayer, "parallel": SharedNormLayer, "sandwich": SandwichNormLayer}


def yarn(base: float, dims: int, s) -> tuple:
    """(divisors of the rotation's frequencies, factor of sine and cosine) of a RotScaling."""
    def pair(turns):                  # the (fractional) pair that turns so often over the original length
        return dims * math.log(s.original / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(pair(s.fast)), 0), min(math.ceil(pair(s.slow)), dims - 1)
    ramp = np.clip((np.arange(dims // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return 1.0 / (ramp / s.factor + (1.0 - ramp)), 0.1 * math.log(s.factor) + 1.0


@dataclass
class _ExpandPlan:
    """The runs of a step that take the prompt attention: `nx` context rows, query blocks of 32 * waves tokens."""
    nx: int
    xmap: torch.Tensor          # [nx] cache slots of the runs' contexts
    blocks: torch.Tensor        # [nblocks][8]
    nblocks: int
    waves: int
    rest: bool                  # some rows attend row by row
    actx: Optional[torch.Tensor]


@dataclass
class _Step:
    T: int
    nruns: int
    block_size: int
    st: int
    plan: Optional[_ExpandPlan] = None
    layer: int = 0              # the layer run: its cache and state (its parts may be another run's)


# runs of at least this many rows expand (below, the latent-space attention's extra products cost less than the expansion
# of the context), as long as their contexts fit the scratch
_EXPAND_RUN = int(os.environ.get("NLS_EXPAND_RUN", "32"))
# runs of at least this many rows take the flash attention of grouped-query layers
_FLASH_RUN = int(os.environ.get("NLS_FLASH_RUN", "16"))
_EXPAND_BYTES = int(os.environ.get("NLS_EXPAND_BYTES", str(4 << 30)))


class StackModel:
    """What the engine drives: step buffers, paged cache rows, state slots and `forward`."""

    format = "safetensors"
    prefill_graphs = False        # (the captured single-prompt prefill of the GGUF families)

    def __init__(self, path: str, device="cuda:0", dtype: torch.dtype = torch.bfloat16, shard: ShardSpec = ShardSpec(),
                 comm=None, ctx: Optional[int] = None):
        self.device = torch.device(device)
        if self.device.type != "cuda":
            raise RuntimeError("stack models run on the GPU kernels only")
        if shard.size > 1:
            raise NotImplementedError("tensor / expert parallelism is not supported for stack models")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("stack models run in bfloat16 or float32")
        K.lib()
        self.path, self.dtype, self.f32 = path, dtype, dtype == torch.float32
        self.shard, self.comm, self.ep = shard, comm, False
        self.reader = r = SafetensorsReader(os.path.join(path, "model.safetensors"))
        self.cfg = cfg = StackConfig.from_dir(path, lambda n: r.shape(n) if n in r else None)
        if ctx is not None:
            cfg.ctx = min(int(ctx), cfg.max_positions) if cfg.max_positions else int(ctx)
        if cfg.d_model > 16384:
            raise ValueError("stack models take widths up to 16384")
        if cfg.n_expert > 512:
            raise ValueError("stack models take up to 512 experts")
        self.weight_bytes = 0
        self._rope = {}
        dev = self.device
        self.embed = r.tensor("embed").to(device=dev, dtype=torch.bfloat16).contiguous()
        self.weight_bytes += self.embed.numel() * 2
        # one layer object per set of weights; self.owners: the one each layer run has; self.passes: the loop's pass that a run
        # starts
        self.owners = [i if cfg.layers[i].weights_of is None else cfg.layers[i].weights_of for i, _ in cfg.order]
        self.passes = [t for _, t in cfg.order]
        layer = LAYERS[cfg.design.norm_place]
        own = {i: layer(self, i, cfg.layers[i]) for i in sorted(set(self.owners))}
        self.layers = [own[o] for o in self.owners]
        self.final_norm = self.norm_weight("final.norm")
        self.head = K.PackedLinear(r.tensor("embed" if cfg.design.tied_head else "head"), self.f32, dev)
        self.weight_bytes += self.head.nbytes
        self.pairs = self.positions = self.loop_in = None
        if cfg.bigram is not None:
            self.pairs = self.table("bigram", cfg.bigram.buckets + 1)
        if cfg.max_positions:
            self.positions = self.table("pos", cfg.max_positions)
        if cfg.loop is not None:
            self.loop_step = r.tensor("loop.step").to(device=dev, dtype=torch.float32).contiguous()
            if tuple(self.loop_step.shape) != (cfg.loop.times, cfg.d_model):
                raise ValueError(f"loop.step: shape {tuple(self.loop_step.shape)}, expected {(cfg.loop.times, cfg.d_model)}")
        if cfg.loop is not None and cfg.design.loop_entry == "product":
            # operand [x | padding | embedding output | padding]
            d, w, ld = cfg.d_model, r.tensor("loop.in").to(dev), K.act_ld(cfg.d_model)
            if tuple(w.shape) != (d, 2 * d):
                raise ValueError(f"loop.in: shape {tuple(w.shape)}, expected {(d, 2 * d)}")
            w = torch.cat([torch.nn.functional.pad(v, (0, ld - d)) for v in (w[:, :d], w[:, d:])], 1)
            self.loop_in = K.PackedLinear(w, self.f32, dev)
            self.weight_bytes += self.loop_in.nbytes
        self.vocab_lo, self.vocab_hi = 0, cfg.vocab

    def table(self, name: str, rows: int) -> torch.Tensor:
        """[rows, width] vectors that are added to the embedding."""
        t = self.reader.tensor(name).to(device=self.device, dtype=torch.bfloat16).contiguous()
        if tuple(t.shape) != (rows, self.cfg.d_model):
            raise ValueError(f"{name}: shape {tuple(t.shape)}, expected {(rows, self.cfg.d_model)}")
        self.weight_bytes += t.numel() * 2
        return t

    def norm_weight(self, name: str) -> torch.Tensor:
        w = self.reader.tensor(name).to(device=self.device, dtype=torch.float32)
        if w.numel() != self.cfg.d_model:
            raise ValueError(f"{name}: {w.numel()} values, expected {self.cfg.d_model}")
        return (w + 1.0 if self.cfg.design.norm_one else w).contiguous()

    # ---- what the engine asks
    @property
    def recurrent(self) -> bool:
        return self.cfg.recurrent

    @property
    def kv_token_bytes(self) -> int:
        return sum(q.cache_width for L in self.layers for q in L.parts) * self.dtype.itemsize

    def n_splits(self, T: int) -> int:
        return 1                      # (each attention layer sizes its own splits)

    def rope(self, base: float, dims: int, scaling=None) -> torch.Tensor:
        key = (base, dims, None if scaling is None else astuple(scaling))
        if key not in self._rope:
            if scaling is None:
                self._rope[key] = rope_table(self.cfg.ctx, dims, base, self.device)
            else:
                factors, gain = yarn(base, dims, scaling)
                self._rope[key] = rope_table(self.cfg.ctx, dims, base, self.device, factors) * gain
        return self._rope[key]

    def kv_cache(self, num_blocks: int, block_size: int = 16):
        """Paged rows of the layer runs that own a cache (one that shares another's weights has its own): {run: rows}."""
        slots = num_blocks * block_size
        return {i: c for i, c in ((i, L.new_caches(slots)) for i, L in enumerate(self.layers)) if c is not None}, None

    def state_pool(self, slots: int):
        """Per-sequence states, f32: {layer run: {name: [slots, n]}} (and "token": the previous token of each slot). A sequence's
        first run (position 0) ignores what its slot holds, so a reused slot needs no clearing."""
        out = {i: {k: torch.zeros(slots, n, dtype=torch.float32, device=self.device)
                   for q in L.parts for k, n in q.state_shapes().items()} for i, L in enumerate(self.layers)}
        if self.pairs is not None:
            out["token"] = torch.zeros(slots, dtype=torch.int32, device=self.device)
        return {i: d for i, d in out.items() if len(d)}

    def step_buffers(self, cap: int, max_seqs: int, max_blocks: int, logit_rows: Optional[int] = None) -> StackBuffers:
        """Step metadata is ONE int32 tensor, as in LlamaModel.step_buffers, with the runs table behind the block tables:
        [ids | pos | slot | tok_seq | ctx_len | use_prev | block_tables | runs]."""
        cfg, dev = self.cfg, self.device
        pad = K.pad_to(cap, 64)
        nb = max_seqs * max_blocks
        meta = torch.zeros(6 * pad + nb + 4 * max_seqs, dtype=torch.int32, device=dev)
        seg = [meta[i * pad:(i + 1) * pad] for i in range(6)]
        f = dict(dtype=torch.float32, device=dev)
        ld = K.act_ld(cfg.d_model)
        nl = min(pad, max(64, max_seqs, logit_rows or 0))
        shared = cfg.design.norm_place in ("shared", "parallel", "sandwich")
        act = lambda: torch.zeros(pad, ld, dtype=self.dtype, device=dev)      # noqa: E731
        b = StackBuffers(
            cap=cap, pad=pad, meta=meta, ids=seg[0], pos=seg[1], slot=seg[2], tok_seq=seg[3], ctx_len=seg[4],
            use_prev=seg[5], block_tables=meta[6 * pad:6 * pad + nb].view(max_seqs, max_blocks),
            runs=meta[6 * pad + nb:].view(max_seqs, 4),
            x=torch.zeros(pad, ld, **f), xb=None if self.f32 or shared else act(), h=act() if shared else None,
            h2=act() if cfg.design.norm_place == "parallel" else None,
            xx=torch.zeros(pad, 2 * ld, dtype=self.dtype, device=dev) if self.loop_in is not None else None,
            y=None if shared else torch.zeros(pad, cfg.d_model, **f), hn=act(),
            logits=torch.zeros(nl, cfg.vocab, **f), next_ids=torch.zeros(pad, dtype=torch.int32, device=dev))
        b.slot.fill_(-1)
        b.runs[:, 2] = -1
        for o, layer in dict(zip(self.owners, self.layers)).items():
            layer.bind(b, o)
        if b.xx is not None:
            b.launches["pass"] = K.LinLaunch([K.Seg(self.loop_in, b.xx, self.slabs(b), slabs=_SLABS, slab_rows=b.slab_rows)])
        cap_epi = dict(epi="softcap", alpha=cfg.softcap) if cfg.softcap else {}
        b.launches["head"] = K.LinLaunch([K.Seg(self.head, b.hn, b.logits, **cap_epi)])
        return b

    # ---- prompt attention: which runs take it
    block_width = K.BLOCK_INTS

    def row_blocks(self, tok_seq, pos, T: int):
        """Host side of a row batch's prompt attention plan, from its staged metadata: (int32 [spans + blocks][8], info), or
        (None, None) when every row attends on its own. Rows of the table: spans (first row, rows, sequence, first
        position, first context row, context, 0, 0), then query blocks (the same, per 32 * waves tokens), longest context
        first."""
        att = [q for L in self.layers for q in L.parts if getattr(q, "attends", False)]
        if not att or any(q.plan_run is None for q in att):
            return None, None
        ts, ps = np.asarray(tok_seq[:T]), np.asarray(pos[:T])
        cut = np.flatnonzero(ts[1:] != ts[:-1]) + 1
        width, least = max(q.plan_bytes for q in att), max(q.plan_run for q in att)
        spans, nx, rows = [], 0, 0
        for a, e in zip(np.concatenate([[0], cut]), np.concatenate([cut, [T]])):
            n, p0 = int(e - a), int(ps[a])
            if n < least or (nx + p0 + n) * width > _EXPAND_BYTES:
                continue
            spans.append((int(a), n, int(ts[a]), p0, nx, p0 + n, 0, 0))
            nx += p0 + n
            rows += n
        if not spans:
            return None, None
        H = max(q.cfg.heads for q in att)
        waves = 8 if H * sum(-(-s[1] // 256) for s in spans) >= 256 else 4
        q = 32 * waves
        blocks = [(s[0] + o, min(q, s[1] - o), s[2], s[3] + o, s[4], 0, 0, 0) for s in spans for o in range(0, s[1], q)]
        blocks.sort(key=lambda v: -(v[3] + v[1]))
        info = dict(nspans=len(spans), nblocks=len(blocks), nx=nx, maxctx=max(s[5] for s in spans), waves=waves,
                    rest=rows < T)
        return np.asarray(spans + blocks, dtype=np.int32), info

    def attention_blocks(self, b: StackBuffers, T: int) -> dict:
        """row_blocks as forward arguments, from a row batch already staged on the device."""
        qb, info = self.row_blocks(b.tok_seq[:T].cpu().numpy(), b.pos[:T].cpu().numpy(), T)
        return {} if qb is None else dict(qblocks=torch.from_numpy(qb).to(self.device), nqb=len(qb), row_info=info)

    def slabs(self, b: StackBuffers) -> torch.Tensor:
        """f32 outputs of a product into the residual, in up to _SLABS blocks of slab_rows rows where K is split."""
        if "slabs" not in b.shared:
            rows = max(b.pad, _SLABS * b.slab_rows)
            b.shared["slabs"] = torch.zeros(rows, self.cfg.d_model, dtype=torch.float32, device=self.device)
        return b.shared["slabs"]

    def grown(self, b: StackBuffers, name: str, rows: int, cols: int, dtype=None) -> torch.Tensor:
        """A [>= rows, cols] scratch that grows (eager row batches only: captured graphs never use it)."""
        key = ("grown", name, cols)
        t = b.shared.get(key)
        if t is None or t.shape[0] < rows:
            b.shared[key] = None
            t = b.shared[key] = torch.zeros(K.pad_to(rows, 1024), cols, dtype=dtype or self.dtype, device=self.device)
        return t

    def _expand_plan(self, b: StackBuffers, qblocks, info: dict, T: int, block_size: int, st: int) -> _ExpandPlan:
        ns = info["nspans"]
        xmap = self.grown(b, "lat.xmap", info["nx"], 1, torch.int32).view(-1)
        actx = None
        if info["rest"]:
            actx = self.grown(b, "lat.actx", b.pad, 1, torch.int32).view(-1)
            actx[:T].copy_(b.ctx_len[:T])
        K.expand_plan(qblocks, ns, info["maxctx"], b.block_tables, block_size, xmap, actx, st)
        return _ExpandPlan(info["nx"], xmap, qblocks[ns:], info["nblocks"], info["waves"], info["rest"], actx)

    # ---- forward
    def _norms(self, b: StackBuffers, i: int) -> dict:
        """What the launch ahead of layer run i leaves for its sublayers, as norm_add's arguments."""
        L = self.layers[i]
        n = dict(out_norm=L.norm1, out=b.h)
        return n if getattr(L, "norm2", None) is None or b.h2 is None else dict(n, out_norm2=L.norm2, out2=b.h2)

    @torch.no_grad()
    def forward(self, b: StackBuffers, kc, vc, T: int, block_size: int, n_split: int = 1,
                logit_rows: Optional[torch.Tensor] = None, n_logits: Optional[int] = None, qblocks=None, nqb: int = 0,
                feed_prev: bool = False, need_logits: bool = True, state=None, nruns: Optional[int] = None,
                row_info: Optional[dict] = None, taps: Optional[list] = None):
        """One step of T rows: logits (of `logit_rows`, or of every row) in b.logits[:n], their greedy ids in
        b.next_ids[:n]. `taps` (a list) receives the residual after every layer."""
        if T < 1 or T > b.pad:
            raise ValueError(f"step of {T} rows, buffers hold {b.pad}")
        cfg = self.cfg
        st = K.stream(self.device)
        step = _Step(T, T if nruns is None else nruns, block_size, st)
        if row_info is not None and qblocks is not None:
            step.plan = self._expand_plan(b, qblocks, row_info, T, block_size, st)
        rms, groups = cfg.design.norm == "rms", cfg.norm_groups
        last = len(self.layers) - 1
        steps = [None if t is None or self.loop_in is not None else self.loop_step[t] for t in self.passes]
        direct = logit_rows is None
        ld = K.act_ld(cfg.d_model)
        more = {}
        if b.xx is not None:                # (the first half ahead of a first pass that no layer precedes)
            more["copies"] = (b.xx[:, ld:], b.xx if self.passes[0] is not None else None)
        if self.pairs is not None:
            bg = cfg.bigram
            more["pairs"] = (self.pairs, bg.buckets, bg.mul_prev, bg.mul_cur, state["token"], b.runs, b.tok_seq)
        if self.positions is not None:
            more["positions"] = (self.positions, b.pos)
        if steps[0] is not None:
            more["add"] = steps[0]
        K.embed(b.ids, self.embed, b.x, b.xb, T, st, prev=(b.next_ids, b.use_prev) if feed_prev else None,
                scale=cfg.embed_scale, **more)
        if b.h is not None and (self.passes[0] is None or steps[0] is not None):
            h = self._norms(b, 0)
            K.row_norm(b.x, None, h["out_norm"], b.h, T, cfg.eps, st, rms=rms, w2=h.get("out_norm2"), out2=h.get("out2"),
                       groups=groups)
        for i, layer in enumerate(self.layers):
            if self.passes[i] is not None and steps[i] is None:
                n = b.launches["pass"].run(T, st)
                K.norm_add(self.slabs(b), None, b.x, None, T, cfg.eps, st, rms=rms, slabs=n, slab_rows=b.slab_rows, keep=False,
                           add=self.loop_step[self.passes[i]], **self._norms(b, i))
            if i == last:
                fin = dict(out_norm=self.final_norm, out=b.hn) if direct else {}
            elif self.passes[i + 1] is not None and steps[i + 1] is None:
                fin = dict(copy=b.xx)
            else:
                fin = self._norms(b, i + 1) if b.h is not None else {}
                if steps[i + 1] is not None:
                    fin["add"] = steps[i + 1]
            step.layer = i
            layer.run(b, self.owners[i], kc, state.get(i) if state else None, step, fin)
            if taps is not None:               # (without the next pass's step, which the layer's last launch adds)
                x = b.x[:T, :cfg.d_model]
                taps.append(x.clone() if i == last or steps[i + 1] is None else x - steps[i + 1])
        n = T
        if not direct:
            n = int(n_logits)
            if n == 0:
                return 0
            K.row_norm(b.x, logit_rows, self.final_norm, b.hn, n, cfg.eps, st, rms=rms, groups=groups)
        if n > b.logits.shape[0]:
            raise ValueError(f"{n} logit rows, buffers hold {b.logits.shape[0]}")
        b.launches["head"].run(n, st)
        K.argmax(b.logits, n, b.next_ids, st)
        return n
