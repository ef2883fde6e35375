"""Device ops of the config-driven decoder stacks: ctypes bindings of `_stack.so` (csrc/stack/*.hip, gfx950).

GPU tensors only: there is no eager form of these ops, a missing library raises. Operands are bf16 (f32 accumulation,
f32 norms / routing / softmax / recurrences) or, for 32-bit models, f32 throughout (f32 MFMA)."""
from __future__ import annotations

import ctypes
import os
from typing import List, Optional

import torch

_PKG = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
LIB_PATH = os.environ.get("NLS_STACK_SO") or os.path.join(_PKG, "_stack.so")

P, I, L, F = ctypes.c_void_p, ctypes.c_int, ctypes.c_long, ctypes.c_float
SEGS = 6
EPI = {"none": 0, "silu": 1, "tanh": 2, "sigmoid": 3, "relu2": 4, "decay": 5, "gate": 6, "rope": 7,
       "geglu": 8, "sigpow": 9, "softcap": 10, "swiglu": 11, "siluglu": 12}
NO_BLOCK = 1 << 30       # LinSeg.cb: output columns are not blocked


class LinSeg(ctypes.Structure):
    """csrc/stack/lin.h LinSeg."""
    _fields_ = [("w", P), ("x", P), ("y", P), ("bias", P), ("gate", P), ("cs", P), ("pos", P), ("rows", P), ("xmap", P),
                ("wstride", L), ("ldx", L), ("ldy", L), ("xgs", L), ("ygs", L), ("yks", L),
                ("N", I), ("nsub", I), ("M", I), ("ng", I), ("epi", I), ("yact", I), ("cb", I), ("cstep", I),
                ("xdiv", I), ("ldg", I), ("half", I), ("alpha", F),
                ("ks", I), ("pad0", I)]


class LinArgs(ctypes.Structure):
    _fields_ = [("s", LinSeg * SEGS), ("tiles", P), ("ntiles", P), ("nseg", I), ("maxtiles", I),
                ("begin", I * (SEGS + 1)), ("nmt", I * SEGS)]


_SIGS = {
    "nls_lin_args_size": [],
    "nls_lin_small": [P, I, I, I, I, P],
    "nls_lin_gemm": [P, I, I, P],
    "nls_stack_embed": [P, P, P, P, I, I, F, P, P, L, I, P, P, L, I, P, I, I, I, P, P, P, P, I, P, P, P],
    "nls_norm_add": [P, L, P, I, L, P, P, L, P, L, P, P, P, P, L, P, I, I, I, F, I, I, I, I, L, P],
    "nls_row_norm": [P, L, P, P, P, P, P, L, P, L, I, I, F, I, I, I, P],
    "nls_poly_norm": [P, L, P, P, L, I, I, F, I, P],
    "nls_attn_rows": [P, P, P, L, P, P, P, P, P, P, L, P, P, L, I, I, I, I, I, I, I, I, I, F, I, P],
    "nls_talk_plain": [P, L, P, P, P, I, I, P, P, I, I, I, I, I, F, I, P, P, L, P, L, I, P],
    "nls_talk_decode": [P, L, P, P, P, I, I, P, P, I, I, I, I, I, I, F, I, P, P, L, P, L, P, L, P, P, P, I, I, I, P],
    "nls_talk_prefill": [P, L, P, P, P, I, I, P, I, I, I, I, I, I, F, I, P, P, L, P, L, P],
    "nls_gqa_attn": [P, L, P, P, P, I, I, P, P, I, I, I, I, I, F, P, L, P, L, P, P, P, I, I, I, I, I, P],
    "nls_gqa_prefill": [P, L, P, P, P, P, I, P, I, P, L, I, I, I, I, F, I, I, I, P],
    "nls_delta_conv": [P, L, P, P, L, P, L, P, L, P, P, I, I, I, I, I, I, I, I, P],
    "nls_delta_scan": [P, P, P, L, P, L, P, L, P, L, P, L, P, P, L, P, L, F, P, L, P, I, I, I, I, I, I, P, P, I, I, P],
    "nls_delta_step": [P, P, P, L, P, L, P, L, P, L, P, P, P, P, I, P, L, P, P, I, L, P, L, P, I, P, P, L, I, I, I, I, F, I, P],
    "nls_gla_scan": [P, P, P, L, P, L, F, P, L, P, P, L, P, L, F, P, L, P, I, I, I, I, I, P, P, I, I, P],
    "nls_gla_step": [P, P, P, L, P, L, P, P, P, I, F, F, P, L, P, I, P, P, L, P, L, P, L, I, I, I, F, I, P],
    "nls_latent_rows": [P, L, I, P, P, L, P, L, I, I, I, P, P, P, P, P, L, I, F, I, P],
    "nls_stack_argmax": [P, L, I, P, I, P],
    "nls_moe_plan": [P, L, I, I, I, I, I, I, I, F, P, P, I, P, P, P, I, P],
    "nls_shift_mix": [P, L, P, P, L, P, L, L, P, P, I, I, I, P],
    "nls_wkv_scan": [P, P, P, L, P, L, P, P, L, P, L, P, L, P, L, I, P, I, I, I, I, P],
    "nls_scan_out": [P, L, P, P, L, P, L, I, I, I, F, I, P],
    "nls_wkv_step": [P, P, P, L, P, L, P, P, L, P, L, P, L, I, P, I, P, P, L, P, L, I, I, F, I, P],
    "nls_expand_plan": [P, I, I, P, I, I, P, P, P],
    "nls_latent_prefill": [P, L, I, P, L, I, P, P, P, L, P, P, I, P, I, P, L, I, I, I, I, I, I, F, P],
    "nls_latent_attn": [P, P, P, P, P, P, I, I, P, P, I, I, I, I, I, F, I, P],
}

_lib = None


def lib():
    global _lib
    if _lib is None:
        if not os.path.exists(LIB_PATH):
            raise RuntimeError(f"HIP kernel library missing: {LIB_PATH} (run `python -m nats_llm_studio_amd.build`)")
        lb = ctypes.CDLL(LIB_PATH)
        for name, args in _SIGS.items():
            fn = getattr(lb, name)
            fn.argtypes = args
            fn.restype = I
        if lb.nls_lin_args_size() != ctypes.sizeof(LinArgs):
            raise RuntimeError("stale _stack.so: LinArgs layout mismatch (rebuild the kernels)")
        _lib = lb
    return _lib


def _check(rc: int, name: str):
    if rc != 0:
        raise RuntimeError(f"{name} failed with code {rc}")


def _p(t: Optional[torch.Tensor]):
    return None if t is None else t.data_ptr()


def stream(dev) -> int:
    return torch.cuda.current_stream(dev).cuda_stream


def pad_to(n: int, m: int) -> int:
    return (n + m - 1) // m * m


def act_ld(n: int) -> int:
    """Row stride of an activation that feeds a linear layer of n inputs: the packed weights' padded K."""
    return pad_to(n, 64)


# ---------------------------------------------------------------------------
# Linear layers
# ---------------------------------------------------------------------------

class PackedLinear:
    """[groups, N, K] weights in the packed layout of csrc/stack/lin.h (1 KiB sub-tiles in MFMA fragment order), bf16
    or f32. A plain matrix is one group; experts and per-head products are stacked groups."""

    def __init__(self, w: torch.Tensor, f32: bool, device):
        if w.dim() == 2:
            w = w[None]
        G, N, K = w.shape
        self.groups, self.N, self.K, self.f32 = G, N, K, f32
        dt, ks, el = (torch.float32, 16, 4) if f32 else (torch.bfloat16, 32, 8)
        Np, Kp = pad_to(N, 16), act_ld(K)
        self.nsub = Kp // ks
        self.data = torch.empty(G, Np * Kp, dtype=dt, device=device)
        step = max(1, (1 << 28) // (Np * Kp))               # groups per conversion pass
        for g0 in range(0, G, step):
            a = w[g0:g0 + step].to(device=device, dtype=dt)
            a = torch.nn.functional.pad(a, (0, Kp - K, 0, Np - N))
            a = a.view(-1, Np // 16, 16, Kp // ks, 4, el).permute(0, 1, 3, 4, 2, 5)
            self.data[g0:g0 + step] = a.reshape(-1, Np * Kp)
        self.wstride = Np * Kp * dt.itemsize

    @property
    def nbytes(self) -> int:
        return self.data.numel() * self.data.element_size()


class Seg:
    """One segment of a LinLaunch. y / x: 2-D buffers (row stride = their stride(0)); ycol / xcol: first column.
    xgs / ygs: column step per group. block = (cb, cstep): output column n -> (n / cb) * cstep + n % cb.
    routed = (entry list, xdiv): the rows are routed entries (x row = entry / xdiv, y row = entry).
    rope = (table, pos, pairs). alpha: constant of the epilogue (sigmoid, sigpow, softcap, swiglu); sigpow: `gate`,
    a vector, gives an exponent per column instead. geglu, swiglu, siluglu: the rows of w alternate gate and up, y has half as many
    columns. slabs: K splits that launches of up to slab_rows rows may use; y holds that many slabs of slab_rows rows, added by
    the caller (LinLaunch.run returns how many were written)."""

    def __init__(self, w: PackedLinear, x: torch.Tensor, y: torch.Tensor, epi: str = "none", ycol: int = 0,
                 xcol: int = 0, xgs: int = 0, ygs: int = 0, block=None, bias=None, gate=None, routed=None, rope=None,
                 yrow: int = 0, xmap: Optional[torch.Tensor] = None, alpha: float = 1.0, slabs: int = 1, slab_rows: int = 0):
        if x.stride(1) != 1 or y.stride(1) != 1:
            raise ValueError("row-major operands")
        if xcol + (0 if routed else (w.groups - 1) * xgs) + act_ld(w.K) > x.stride(0):
            raise ValueError(f"x rows ({x.stride(0)}) do not cover the padded K of {w.K} inputs")
        if x.dtype != w.data.dtype:
            raise TypeError(f"activations must be {w.data.dtype}, got {x.dtype}")
        if (xcol * x.element_size()) % 16 or (x.stride(0) * x.element_size()) % 16 or (xgs * x.element_size()) % 16:
            raise ValueError("activation rows must be 16-byte aligned")
        self.w, self.y, self.x = w, y, x
        self.rows_cap = min(x.shape[0] * (routed[1] if routed else 1), y.shape[0] - yrow)
        if xmap is not None:               # x row of row m: xmap[m] (the caller keeps the entries inside x)
            self.rows_cap = min(xmap.numel(), y.shape[0] - yrow)
        s = self.s = LinSeg()
        s.w = w.data.data_ptr()
        s.x = x.data_ptr() + xcol * x.element_size()
        s.y = y.data_ptr() + (yrow * y.stride(0) + ycol) * y.element_size()
        s.bias, s.gate = _p(bias), _p(gate)
        s.ldg = gate.stride(0) if gate is not None else 0
        s.wstride, s.ldx, s.ldy, s.xgs, s.ygs = w.wstride, x.stride(0), y.stride(0), xgs, ygs
        s.N, s.nsub, s.ng, s.epi = w.N, w.nsub, w.groups, EPI[epi]
        s.yact = int(y.dtype != torch.float32)
        s.cb, s.cstep = block if block else (NO_BLOCK, 0)
        s.xdiv = 1
        if routed:
            s.rows, s.xdiv = routed[0].data_ptr(), routed[1]
        if rope:
            s.cs, s.pos, s.half = rope[0].data_ptr(), rope[1].data_ptr(), rope[2]
        s.xmap = _p(xmap)
        s.alpha = alpha
        if slabs * slab_rows > y.shape[0]:
            raise ValueError("y does not hold the slabs")
        s.ks, self.slabs, self.slab_rows = 1, slabs, slab_rows
        s.yks = slab_rows * y.stride(0)
        self.keep = (bias, gate, routed, rope, xmap)


# (weight rows, rows) of lin_gemm's configs
GEMM_TILES = ((64, 64), (128, 64), (128, 128), (256, 128), (256, 256), (64, 64), (192, 128))


# relative multiply rates of the tiles: (up to so many workgroups, below, above); the small tiles run two or more to a CU
GEMM_RATE = {4: (0, 0.96, 0.96), 3: (0, 1.0, 1.0), 6: (0, 0.96, 0.96), 2: (256, 0.47, 0.72),
             1: (512, 0.5, 0.63), 0: (1024, 0.45, 0.55)}


class LinLaunch:
    """A launch of up to SEGS independent linear layers, bound to its buffers once (only the row count and the launch
    config change from step to step)."""

    def __init__(self, segs: List[Seg], plan: "MoePlan" = None):
        self.segs, self.plan = segs, plan
        self.f32 = int(segs[0].w.f32)
        self.a = LinArgs()
        for i, s in enumerate(segs):
            self.a.s[i] = s.s
        self.a.nseg = len(segs)
        if plan is not None:
            self.a.tiles, self.a.ntiles = plan.tiles.data_ptr(), plan.ntiles.data_ptr()
        self._cfg = {}

    def _tiles(self, bn: int, bm: int, M: int) -> int:
        """Workgroups of a launch with bn x bm tiles."""
        n = 0
        for s in self.segs:
            nt = (s.w.N + bn - 1) // bn
            n += nt * (self.plan.expect_tiles(M, bm) if s.s.rows else s.w.groups * ((M + bm - 1) // bm))
        return n

    def config(self, M: int):
        """(False, mt, nw, rt): few-row kernel with mt activation tiles, nw waves and rt weight tiles per workgroup; or
        (True, c): GEMM config c."""
        if self.plan is not None:
            bm = self.plan.bm(M)
            if bm == 16:
                return False, 1, (4 if self._tiles(16, 16, M) >= 1536 else 8), 1
            if bm == 64:
                return True, 0
            return True, (3 if self._tiles(256, 128, M) >= 224 else 2)
        n16, n64 = self._tiles(16, 16, M), self._tiles(64, 64, M)
        ns = max(s.w.nsub for s in self.segs)
        if M <= 16:
            if M > 8 and n16 >= 1024:
                return False, 1, 4, 2
            return False, 1, (4 if ns <= 16 else 8 if n16 >= 320 or ns <= 32 else 16), 1
        if n16 <= 64:                     # a router's few outputs: split K over a workgroup's waves
            return False, 1, 16, 1
        if M <= 64:
            if n64 >= 250:
                return True, 0
            return False, 2, (4 if ns <= 16 else 8), (2 if M > 32 or n16 >= 640 else 1)
        if ns <= 4:                       # a step or two of K: all epilogue
            return True, (0 if M <= 2048 else 1)
        if n64 < 96 and n16 <= 1024:
            return False, 1, 16, 1
        if M > 512:
            cand = GEMM_RATE
        elif self._tiles(256, 128, M) >= 120:
            cand = (3, 6)
        else:
            return True, (5 if n64 <= 256 else 0)

        # rounds of 256 workgroups times a tile's cost
        def cost(c):
            n, (few, lo, hi) = self._tiles(*GEMM_TILES[c], M), GEMM_RATE[c]
            return -(-n // 256) * GEMM_TILES[c][0] * GEMM_TILES[c][1] / (lo if n <= few else hi)
        return True, min(cand, key=cost)

    def split_config(self, M: int):
        """(config, K splits) of a launch that may split K: about 512 workgroups of 64 x 64 tiles, or 256 of 256 x 128."""
        n16 = self._tiles(16, 16, M)
        if M <= 16:
            rt = 1 if M <= 8 else 2
            return (False, 1, 8, rt), -(-512 * rt // (2 * n16)) if M > 8 else -(-512 // n16)
        if M <= 32:
            return (False, 2, 4, 4 if n16 >= 256 else 2), 8
        big, small = self._tiles(256, 128, M), self._tiles(64, 64, M)
        if M > 128 and big * 8 >= 256:
            return (True, 3), -(-256 // big)
        return (True, 0), -(-512 // small)

    def run(self, M: int, st: int) -> int:
        """Returns the slabs of output rows that were written (1 unless a segment may split K)."""
        if self.plan is not None:
            self.a.maxtiles = self.plan.max_tiles(M)
        for i, s in enumerate(self.segs):
            if (M * self.plan.top if s.s.rows else M) > s.rows_cap:
                raise ValueError(f"linear launch: {M} rows but the buffers hold {s.rows_cap}")
            self.a.s[i].M = M
        cfg = self._cfg.get(M)
        if cfg is None:
            if len(self._cfg) > 4096:
                self._cfg.clear()
            s = self.segs[0]
            if s.slabs > 1 and len(self.segs) == 1 and M <= s.slab_rows and s.w.nsub >= 64:
                cfg, ks = self.split_config(M)
                cfg = cfg, max(1, min(ks, s.slabs, s.w.nsub // 16))
            else:
                cfg = self.config(M), 1
            self._cfg[M] = cfg
        cfg, ks = cfg
        self.a.s[0].ks = ks
        if cfg[0]:
            _check(lib().nls_lin_gemm(ctypes.byref(self.a), self.f32, cfg[1], st), "nls_lin_gemm")
        else:
            _check(lib().nls_lin_small(ctypes.byref(self.a), self.f32, *cfg[1:], st), "nls_lin_small")
        return ks


class MoePlan:
    """Expert choice and routed-entry lists of one step (csrc/stack/stack_ops.hip moe_plan_kernel), shared by the layers
    of a step. Scores: sigmoid of the router logits, or their softmax; the `keep` groups with the largest score (the sum of
    their `group_best` best) of `groups` stay eligible; a chosen expert's weight is score * scale."""

    def __init__(self, cap: int, experts: int, top: int, groups: int, keep: int, scale: float, device, score: str = "sigmoid",
                 group_best: int = 2):
        self.softmax, self.group_best = {"sigmoid": 0, "softmax": 1}[score], group_best
        self.experts, self.top, self.groups, self.keep, self.scale = experts, top, groups, keep, scale
        i32 = dict(dtype=torch.int32, device=device)
        self.topw = torch.zeros(cap * top, dtype=torch.float32, device=device)
        self.sel = torch.zeros(cap * top, **i32)
        self.rows = torch.zeros(cap * top, **i32)
        self.tiles = torch.zeros(self.max_tiles(cap, 16), 4, **i32)
        self.ntiles = torch.zeros(4, **i32)

    def bm(self, T: int) -> int:
        """Rows per tile of the expert products at T tokens."""
        avg = T * self.top / self.experts
        return 16 if avg <= 6 else (64 if avg <= 96 else 128)

    def max_tiles(self, T: int, bm: Optional[int] = None) -> int:
        bm = bm or self.bm(T)
        n = T * self.top
        return max(1, min(n, self.experts + n // bm))

    def expect_tiles(self, T: int, bm: int) -> int:
        """About how many tiles T tokens make (launch rules)."""
        n = T * self.top
        return max(1, min(n, self.experts), n // bm)

    def run(self, z: torch.Tensor, T: int, st: int):
        _check(lib().nls_moe_plan(z.data_ptr(), z.stride(0), T, self.experts, self.top, self.groups, self.keep,
                                  self.softmax, self.group_best, self.scale, self.topw.data_ptr(), self.sel.data_ptr(), self.bm(T),
                                  self.rows.data_ptr(), self.tiles.data_ptr(), self.ntiles.data_ptr(),
                                  self.max_tiles(T), st), "nls_moe_plan")


# ---------------------------------------------------------------------------
# Row kernels
# ---------------------------------------------------------------------------

def embed(ids, table: torch.Tensor, x: torch.Tensor, xb: Optional[torch.Tensor], T: int, st: int, prev=None,
          scale: float = 1.0, copies=(), pairs=None, positions=None, add: Optional[torch.Tensor] = None):
    """x = table[id] * scale (xb: its bf16 rounding). copies: up to two more of x in the activation type, of one row stride.
    pairs = (table, buckets, mul_prev, mul_cur, previous token of each slot, runs, tok_seq): plus the row of the token pair, and
    the slots' tokens move on. positions = (table, pos): plus the position's row. add: plus a vector."""
    nx, up = prev if prev is not None else (None, None)
    c0, c1 = (tuple(copies) + (None, None))[:2]
    pt, nb, mp, mc, pv, runs, seq = pairs if pairs is not None else (None, 0, 0, 0, None, None, None)
    tab, pos = positions if positions is not None else (None, None)
    _check(lib().nls_stack_embed(ids.data_ptr(), _p(nx), _p(up), table.data_ptr(), table.shape[0], table.shape[1], scale,
                                 x.data_ptr(), _p(xb), x.stride(0), T, _p(c0), _p(c1), c0.stride(0) if c0 is not None else 0,
                                 int(c0 is not None and c0.dtype == torch.float32), _p(pt), nb, mp, mc, _p(pv), _p(runs), _p(seq),
                                 _p(tab), tab.shape[0] if tab is not None else 0, _p(pos), _p(add), st), "nls_stack_embed")


def norm_add(y: torch.Tensor, w: Optional[torch.Tensor], x: torch.Tensor, xb: Optional[torch.Tensor], T: int, eps: float,
             st: int, plan: Optional[MoePlan] = None, shared_row0: int = -1, out_norm: Optional[torch.Tensor] = None,
             out: Optional[torch.Tensor] = None, rms: bool = False, slabs: int = 1, slab_rows: int = 0, out_norm2=None, out2=None,
             keep: bool = True, add: Optional[torch.Tensor] = None, groups: int = 1):
    """x[:T] += norm(y) * w, or += y without w (xb: a copy in the activation type); y may be the sum of `slabs` blocks of
    slab_rows rows. With `plan`, y holds the routed experts' rows (token-major) and from row `shared_row0` on the shared
    expert's, combined first. out = norm(x) * out_norm (what the next sublayers read, or the model's last norm), out2 the same
    with out_norm2. norm: layer norm, or RMS (of `groups` equal parts of a row each on its own). add: a vector that comes on top of
    x; keep False: the old x is left out."""
    D = y.shape[1] if w is None else w.numel()
    typed = out if out is not None else xb
    if out2 is not None and out2.stride(0) != out.stride(0):
        raise ValueError("norm_add: equal row strides of the outputs")
    _check(lib().nls_norm_add(y.data_ptr(), y.stride(0), _p(plan.topw) if plan else None, plan.top if plan else 0,
                              shared_row0, _p(w), x.data_ptr(), x.stride(0), _p(xb), xb.stride(0) if xb is not None else 0,
                              _p(out_norm), _p(out), _p(out_norm2), _p(out2), out.stride(0) if out is not None else 0, _p(add),
                              int(keep), D, T, eps, int(typed is not None and typed.dtype == torch.float32), int(rms), groups, slabs,
                              slab_rows * y.stride(0), st), "nls_norm_add")


def row_norm(x: torch.Tensor, rows: Optional[torch.Tensor], w: torch.Tensor, out: torch.Tensor, n: int, eps: float,
             st: int, rms: bool = False, w2=None, out2=None, gate: Optional[torch.Tensor] = None, groups: int = 1):
    """out[i] = norm(x[rows[i]]) * w (rows None: row i) (* gate[i]): layer norm, or RMS (of `groups` parts each on its own). out2: the
    same with w2."""
    if (out2 is not None and out2.stride(0) != out.stride(0)) or (gate is not None and gate.dtype != out.dtype):
        raise ValueError("row_norm: equal row strides of the outputs, a gate of their type")
    _check(lib().nls_row_norm(x.data_ptr(), x.stride(0), _p(rows), w.data_ptr(), out.data_ptr(), _p(w2), _p(out2), out.stride(0),
                              _p(gate), gate.stride(0) if gate is not None else 0, w.numel(), n, eps,
                              int(out.dtype == torch.float32), int(rms), groups, st), "nls_row_norm")


def poly_norm(z: torch.Tensor, act: torch.Tensor, out: torch.Tensor, N: int, T: int, eps: float, st: int):
    """out = a rms(z) + b rms(z^2) + c rms(z^3) + e over rows of N columns, powers by element; act: (a, b, c, e)."""
    if z.dtype != out.dtype or act.numel() != 4 or N > min(z.stride(0), out.stride(0)):
        raise ValueError("poly_norm: equal types, rows of N columns, four factors")
    _check(lib().nls_poly_norm(z.data_ptr(), z.stride(0), act.data_ptr(), out.data_ptr(), out.stride(0), N, T, eps,
                               int(out.dtype == torch.float32), st), "nls_poly_norm")


def argmax(logits: torch.Tensor, n: int, out: torch.Tensor, st: int):
    _check(lib().nls_stack_argmax(logits.data_ptr(), logits.stride(0), logits.shape[1], out.data_ptr(), n, st),
           "nls_stack_argmax")


def latent_rows(dq, wq, cq, dkv, wc, R: int, Rp: int, rot: int, cs, pos, slot, cache, T: int, eps: float, st: int):
    """cq = RMSNorm(dq) * wq; with `dkv`: the tokens' cache rows [RMSNorm(dkv[:R]) * wc | rotated dkv[R:]]."""
    _check(lib().nls_latent_rows(dq.data_ptr(), dq.stride(0), wq.numel(), wq.data_ptr(), cq.data_ptr(), cq.stride(0),
                                 _p(dkv), dkv.stride(0) if dkv is not None else 0, R, Rp, rot, _p(wc), cs.data_ptr(),
                                 pos.data_ptr(), slot.data_ptr(), _p(cache), cache.stride(0) if cache is not None else 0,
                                 T, eps, int(cq.dtype == torch.float32), st), "nls_latent_rows")


LATENT_TILES = (1, 2, 3, 4, 6, 8, 12, 16)     # padded latent widths / 64 the attention kernels are built for


def latent_pad(R: int) -> int:
    for n in LATENT_TILES:
        if R <= 64 * n:
            return 64 * n
    raise ValueError(f"latent width {R} > {64 * LATENT_TILES[-1]}")


def latent_head_groups(H: int, Rp: int) -> int:
    """Workgroups a (token, split) of latent_attention takes: 16 heads each, or 32 (csrc/stack/latent_attn.hip launch_r)."""
    return -(-H // (32 if H > 16 and Rp < 1024 else 16))


def rot_pad(rot: int) -> int:
    if rot > 128:
        raise ValueError(f"rotated width {rot} > 128")
    return 64 if rot <= 64 else 128


def latent_attention(q, cache, out, part, block_tables, block_size: int, tok_seq, ctx_len, T: int, H: int, ns: int,
                     Rp: int, rp: int, scale: float, st: int):
    po, pm = part if part is not None else (None, None)
    if ns > 1 and (po.numel() < T * H * ns * Rp or pm.numel() < T * H * ns * 2):
        raise ValueError("latent_attention: split workspace too small")
    _check(lib().nls_latent_attn(q.data_ptr(), cache.data_ptr(), out.data_ptr(), _p(po), _p(pm), block_tables.data_ptr(),
                                 block_tables.stride(0), block_size, tok_seq.data_ptr(), ctx_len.data_ptr(), T, H, ns,
                                 Rp, rp, scale, int(q.dtype == torch.float32), st), "nls_latent_attn")


BLOCK_INTS = 8           # int32 words per span / query block of the row plan (StackModel.row_blocks)
EXPAND_UNITS = {"key": (32, 64, 128), "rot": (32, 64), "value": (32, 64, 128)}      # per-head widths of latent_prefill


def expand_width(kind: str, n: int) -> Optional[int]:
    return next((w for w in EXPAND_UNITS[kind] if n <= w), None)


def expand_plan(spans, nspans: int, maxctx: int, block_tables, block_size: int, xmap, actx, st: int):
    """xmap: cache slots of the spans' contexts; actx (optional): key counts of the rows, cleared inside the spans."""
    _check(lib().nls_expand_plan(spans.data_ptr(), nspans, maxctx, block_tables.data_ptr(), block_tables.stride(0),
                                 block_size, xmap.data_ptr(), _p(actx), st), "nls_expand_plan")


def latent_prefill(qn, qns: int, q, Rp: int, qrs: int, kx, vx, cache, xmap, blocks, nblocks: int, waves: int, gate, out,
                   H: int, dku: int, dr: int, dv: int, vdim: int, scale: float, st: int):
    """Causal attention of query blocks over expanded keys / values; the rotated parts sit at column Rp of q and cache."""
    _check(lib().nls_latent_prefill(qn.data_ptr(), qn.stride(0), qns, q.data_ptr() + Rp * q.element_size(), q.stride(0), qrs,
                                    kx.data_ptr(), vx.data_ptr(), cache.data_ptr() + Rp * cache.element_size(),
                                    cache.stride(0), xmap.data_ptr(), blocks.data_ptr(), nblocks, gate.data_ptr(),
                                    gate.stride(0), out.data_ptr(), out.stride(0), H, dku, dr, dv, vdim, waves, scale, st),
           "nls_latent_prefill")


def shift_mix(x, mu, prev, out: torch.Tensor, runs, tok_seq, T: int, st: int):
    """out [mixes, rows, ld]: x + (previous token's x - x) * mu[s]; `prev` [slots, D] precedes each run's first row."""
    _check(lib().nls_shift_mix(x.data_ptr(), x.stride(0), mu.data_ptr(), prev.data_ptr(), prev.stride(0), out.data_ptr(),
                               out.stride(1), out.stride(0), runs.data_ptr(), tok_seq.data_ptr(), mu.shape[1], T,
                               int(out.dtype == torch.float32), st), "nls_shift_mix")


def wkv_scan(r, k, v, w, u, o, state, x, prev, runs, nruns: int, H: int, D: int, st: int):
    """The recurrence over each run's tokens; state [slots, H * D * D] and prev [slots, width] are carried on."""
    _check(lib().nls_wkv_scan(r.data_ptr(), k.data_ptr(), v.data_ptr(), r.stride(0), w.data_ptr(), w.stride(0),
                              u.data_ptr(), o.data_ptr(), o.stride(0), state.data_ptr(), state.stride(0), x.data_ptr(),
                              x.stride(0), prev.data_ptr(), prev.stride(0), prev.shape[1], runs.data_ptr(), nruns, H, D,
                              int(r.dtype == torch.float32), st), "nls_wkv_scan")


def wkv_step(r, k, v, w, u, state, x, prev, runs, nruns: int, norm, gate, out, H: int, D: int, eps: float, st: int):
    """wkv_scan and wkv_out of runs of one token each."""
    _check(lib().nls_wkv_step(r.data_ptr(), k.data_ptr(), v.data_ptr(), r.stride(0), w.data_ptr(), w.stride(0), u.data_ptr(),
                              state.data_ptr(), state.stride(0), x.data_ptr(), x.stride(0), prev.data_ptr(),
                              prev.stride(0), prev.shape[1], runs.data_ptr(), nruns, norm.data_ptr(), gate.data_ptr(),
                              gate.stride(0), out.data_ptr(), out.stride(0), H, D, eps, int(out.dtype == torch.float32),
                              st), "nls_wkv_step")


def scan_out(o, norm, gate, out, H: int, D: int, T: int, eps: float, st: int):
    """out = (o / rms(o) per head of D columns) * norm * gate."""
    _check(lib().nls_scan_out(o.data_ptr(), o.stride(0), norm.data_ptr(), gate.data_ptr(), gate.stride(0), out.data_ptr(),
                              out.stride(0), H, D, T, eps, int(out.dtype == torch.float32), st), "nls_scan_out")


def gla_shape(T: int, nruns: int, H: int, V: int):
    """(segments, groups of 64 value columns per workgroup) of a gla_scan launch: two workgroups per CU from segments of at
    least 64 tokens, unless whole runs already give one."""
    nt = 1 if V <= 64 else 2
    wgs = H * -(-V // (64 * nt)) * nruns
    return 1 if wgs >= 256 else max(1, min(-(-512 // wgs), (T - nruns + 1) // 64, 16)), nt


def gla_scan(q, k, v, a, qscale: float, o, norm, gate, out, state, runs, nruns: int, H: int, D: int, V: int, eps: float, shape,
             seg, st: int):
    """Gated linear attention over each run's tokens: q, k [rows, H * D], v [rows, H * V] of one buffer (equal strides), decays
    a; state [slots, H * D * V] is carried on. With `out` (a head's columns fit a workgroup): its norm, `norm` and `gate`
    applied, else the plain outputs in `o` (scan_out follows). shape: gla_shape; seg: (states, decay products) scratch of its
    segments."""
    nseg, nt = shape
    if nseg > 1 and (seg[0].numel() < nruns * nseg * H * D * V or seg[1].numel() < nruns * nseg * H * D):
        raise ValueError("gla_scan: segment scratch too small")
    s0, s1 = seg if nseg > 1 else (None, None)
    f = out is not None
    _check(lib().nls_gla_scan(q.data_ptr(), k.data_ptr(), v.data_ptr(), q.stride(0), a.data_ptr(), a.stride(0), qscale,
                              _p(o), o.stride(0) if o is not None else 0, norm.data_ptr() if f else None,
                              gate.data_ptr() if f else None, gate.stride(0) if f else 0, _p(out), out.stride(0) if f else 0,
                              eps, state.data_ptr(), state.stride(0), runs.data_ptr(), nruns, H, D, V, nseg, _p(s0), _p(s1), nt,
                              int(q.dtype == torch.float32), st), "nls_gla_scan")


def gla_step(q, k, v, a, gate_in, qscale: float, state, runs, nruns: int, norm, gate, out, H: int, D: int, V: int, eps: float,
             st: int, o=None):
    """gla_scan of runs of one token each (V a multiple of 4), with the norm and gate, or (norm None) the plain outputs in `o`.
    Decays `a`, or (None) from gate_in = (low-rank gate input, a2, bias, exponent): sigmoid(a2 low + bias) ^ exponent."""
    lo, a2, b, ia = gate_in if a is None else (None, None, None, 0.0)
    y = out if norm is not None else o
    _check(lib().nls_gla_step(q.data_ptr(), k.data_ptr(), v.data_ptr(), q.stride(0), _p(a), a.stride(0) if a is not None else 0,
                              _p(lo), _p(a2), _p(b), a2.shape[1] if a2 is not None else 0, ia, qscale, state.data_ptr(),
                              state.stride(0), runs.data_ptr(), nruns, _p(norm), _p(gate),
                              gate.stride(0) if gate is not None else 0, _p(out), out.stride(0) if out is not None else 0, _p(o),
                              o.stride(0) if o is not None else 0, H, D, V, eps, int(q.dtype == torch.float32), st),
           "nls_gla_step")


# ---------------------------------------------------------------------------
# Delta rule
# ---------------------------------------------------------------------------

def delta_conv(z, w, y, fac, state, runs, tok_seq, T: int, nruns: int, H: int, G: int, D: int, V: int, st: int):
    """y = silu(causal convolution of z) per channel, [q: G * D | k: G * D | v: H * V]; w f32 [channels, taps]; the last taps - 1
    inputs are carried in state [slots, (taps - 1) * channels] (None for one tap). fac [rows, 2 G]: what makes the heads of q
    (times D^-1/2) and k unit vectors."""
    _check(lib().nls_delta_conv(z.data_ptr(), z.stride(0), w.data_ptr(), y.data_ptr(), y.stride(0), fac.data_ptr(), fac.stride(0),
                                _p(state), state.stride(0) if state is not None else 0, runs.data_ptr(), tok_seq.data_ptr(), T,
                                nruns, H, G, D, V, w.shape[1], int(z.dtype == torch.float32), st), "nls_delta_conv")


def delta_shape(T: int, nruns: int, H: int, D: int, V: int):
    """(segments, groups of 64 value columns per workgroup) of a delta_scan launch. Segments cost a second pass over the tokens
    with D more columns, so they start where whole runs fill less than half the CUs, and stay longer."""
    nt = 1 if V <= 64 else 2
    wgs = H * -(-V // (64 * nt)) * nruns
    return 1 if wgs >= 128 else max(1, min(-(-256 // wgs), (T - nruns + 1) // 128, 16)), nt


def delta_scan(q, k, v, fac, beta, a, o, norm, gate, out, state, runs, nruns: int, H: int, G: int, D: int, V: int, eps: float,
               shape, seg, st: int):
    """The delta rule over each run's tokens: q, k [rows, G * D], v [rows, H * V] of one buffer, the factors of delta_conv, beta
    [rows, H], decays a [rows, H * D]; otherwise as gla_scan. seg: (states, matrices) scratch of the segments."""
    nseg, nt = shape
    if nseg > 1 and (seg[0].numel() < nruns * nseg * H * D * V or seg[1].numel() < nruns * nseg * H * D * D):
        raise ValueError("delta_scan: segment scratch too small")
    s0, s1 = seg if nseg > 1 else (None, None)
    f = out is not None
    _check(lib().nls_delta_scan(q.data_ptr(), k.data_ptr(), v.data_ptr(), q.stride(0), fac.data_ptr(), fac.stride(0),
                                beta.data_ptr(), beta.stride(0), a.data_ptr(), a.stride(0), _p(o), o.stride(0) if o is not None else 0,
                                norm.data_ptr() if f else None, gate.data_ptr() if f else None, gate.stride(0) if f else 0, _p(out),
                                out.stride(0) if f else 0, eps, state.data_ptr(), state.stride(0), runs.data_ptr(), nruns, H, G, D,
                                V, nseg, _p(s0), _p(s1), nt, int(q.dtype == torch.float32), st), "nls_delta_scan")


def delta_step(q, k, v, fac, beta, a, decay_in, gate, gate_in, ldz: int, state, runs, nruns: int, norm, out, H: int, G: int, D: int,
               V: int, eps: float, st: int):
    """delta_scan of runs of one token each (V a multiple of 4), with the norm and gate. Decays a, or (None) from decay_in =
    (low-rank input, a2, bias, exponent per channel): sigmoid(a2 low + bias) ^ exponent. The gate, or (None) from gate_in =
    (low-rank input, g2): sigmoid(g2 low). ldz: row stride of the low-rank inputs."""
    lo, a2, b, rate = decay_in if a is None else (None, None, None, None)
    lg, g2 = gate_in if gate is None else (None, None)
    _check(lib().nls_delta_step(q.data_ptr(), k.data_ptr(), v.data_ptr(), q.stride(0), fac.data_ptr(), fac.stride(0),
                                beta.data_ptr(), beta.stride(0), _p(a), a.stride(0) if a is not None else 0, _p(lo), _p(a2), _p(b),
                                _p(rate), a2.shape[1] if a2 is not None else 0, _p(gate),
                                gate.stride(0) if gate is not None else 0, _p(lg), _p(g2), g2.shape[1] if g2 is not None else 0, ldz,
                                state.data_ptr(), state.stride(0), runs.data_ptr(), nruns, norm.data_ptr(), out.data_ptr(),
                                out.stride(0), H, G, D, V, eps, int(out.dtype == torch.float32), st), "nls_delta_step")


# ---------------------------------------------------------------------------
# Grouped-query attention
# ---------------------------------------------------------------------------

HEAD_WIDTHS = (32, 64, 128, 256)      # padded head widths of the MFMA attention kernels


def head_pad(D: int):
    """(padded head width, MFMA kernels): other widths run on the plain kernel, padded for its 16-byte loads."""
    for w in HEAD_WIDTHS:
        if D <= w:
            return w, True
    if D > 1024:
        raise ValueError(f"attention head width {D} > 1024")
    return pad_to(D, 32), False


def attn_groups(H: int, G: int) -> int:
    """Workgroups a (token, split) of gqa_attention takes."""
    return G * -(-(H // G) // 16)


def attn_rows(q, k, v, qn, kn, cs, pos, slot, qo, kc, vc, T: int, H: int, G: int, D: int, Dp: int, rot: int, eps: float, st: int,
              V: Optional[int] = None, head_norm: bool = False, key_tiles: bool = False):
    """Norm over the whole q and k projections (qn, kn: weights or None), rotation of the first `rot` columns of each head (cs
    None: none), then (head_norm) an RMS norm of each head of queries and keys on its own; queries to qo, keys and (as projected, V
    columns per head) values to the tokens' cache rows. q, k, v: f32 with one row stride. key_tiles: 16 slots of the key cache are a
    tile [G][Dp / 8][16][8] (slots in whole tiles)."""
    if key_tiles and kc.shape[0] % KEY_TILE:
        raise ValueError("attn_rows: a key cache of whole tiles")
    _check(lib().nls_attn_rows(q.data_ptr(), k.data_ptr(), v.data_ptr(), q.stride(0), _p(qn), _p(kn), _p(cs),
                               pos.data_ptr(), slot.data_ptr(), qo.data_ptr(), qo.stride(0), kc.data_ptr(), vc.data_ptr(),
                               kc.stride(0), T, H, G, D, D if V is None else V, Dp, rot, int(head_norm),
                               int(key_tiles), eps,
                               int(qo.dtype == torch.float32), st),
           "nls_attn_rows")


def gqa_attention(q, kc, vc, gate, out, part, block_tables, block_size: int, tok_seq, ctx_len, T: int, H: int, G: int, Dp: int,
                  mfma: bool, ns: int, scale: float, st: int, window: int = 0, keep: int = 0, sink: bool = False):
    """Row-by-row attention (decoded tokens, short runs); a head gate (or None) is applied to the output. part: (partial
    outputs, (max, sum) pairs, ticket counters) of `ns` splits. window > 0: the newest `window` keys and the first `keep`;
    sink: the softmax's denominator holds one more, a score of 0 without a value."""
    po, pm, cnt = part
    if ns > 1 and (po.numel() < T * H * ns * Dp or pm.numel() < T * H * ns * 2 or cnt.numel() < T * attn_groups(H, G)):
        raise ValueError("gqa_attention: split workspace too small")
    _check(lib().nls_gqa_attn(q.data_ptr(), q.stride(0), kc.data_ptr(), vc.data_ptr(), block_tables.data_ptr(),
                              block_tables.stride(0), block_size, tok_seq.data_ptr(), ctx_len.data_ptr(), T, H, G, Dp, ns,
                              scale, _p(gate), gate.stride(0) if gate is not None else 0, out.data_ptr(), out.stride(0),
                              po.data_ptr(), pm.data_ptr(), cnt.data_ptr(), window, keep, int(sink), int(not mfma),
                              int(q.dtype == torch.float32), st), "nls_gqa_attn")


def gqa_prefill(q, kc, vc, xmap, blocks, nblocks: int, waves: int, gate, out, H: int, G: int, Dp: int, scale: float, st: int,
                window: int = 0, keep: int = 0, sink: bool = False):
    """Causal attention of query blocks over their sequences' paged keys and values (gate, window, keep, sink: as
    gqa_attention)."""
    _check(lib().nls_gqa_prefill(q.data_ptr(), q.stride(0), kc.data_ptr(), vc.data_ptr(), xmap.data_ptr(), blocks.data_ptr(),
                                 nblocks, _p(gate), gate.stride(0) if gate is not None else 0, out.data_ptr(), out.stride(0), H, G,
                                 Dp, waves, scale, window, keep, int(sink), st), "nls_gqa_prefill")


# ---------------------------------------------------------------------------
# Attention with mixed heads
# ---------------------------------------------------------------------------

KEY_TILE = 16                           # slots of a key tile
TALK_WIDTHS = (32, 64, 128)             # padded head widths of the prompt kernel, which takes up to 32 heads
TALK_SCRATCH = 256 << 20                # bytes of scores that a decode launch may hold


class TalkPlan:
    """Kernels and scratch sizes of an attention whose heads' softmax weights are mixed, heads padded to Dp columns. The MFMA kernels
    read keys in tiles of 16 slots (attn_rows: key_tiles), the plain one rows."""

    def __init__(self, H: int, G: int, Dp: int, window: int, ctx: int, f32: bool, device, scale: float = 1.0):
        self.H, self.G, self.Dp, self.window = H, G, Dp, window
        self.mfma = not f32 and Dp in HEAD_WIDTHS and H <= 128
        self.prefill = self.mfma and H <= 32 and Dp in TALK_WIDTHS and scale > 0
        self.groups, self.hs = attn_groups(H, G), pad_to(H, 8)
        self.ks = pad_to(min(window or ctx, ctx), 32) + 32              # keys of a row, from a multiple of 32 on
        self.device = device

    def matrix(self, talk: torch.Tensor) -> torch.Tensor:
        """The [H, H] matrix as the kernels read it."""
        if not self.mfma:
            return talk.to(device=self.device, dtype=torch.float32).contiguous()
        n = pad_to(self.H, 32) if self.H <= 64 else 128
        out = torch.zeros(n, n, dtype=torch.bfloat16, device=self.device)
        out[:self.H, :self.H] = talk.to(self.device)
        return out

    def rows(self, cap: int) -> int:
        """Rows of a decode launch."""
        return max(1, min(cap, TALK_SCRATCH // (4 * self.ks * self.hs)))

    def splits(self, T: int):
        """(splits of the scores, of the values, waves of a workgroup of the latter) at T rows."""
        n = T * self.groups
        ns1 = max(1, min(64, 2048 // n))
        if n >= 1024 or self.Dp > 128:
            return ns1, max(1, min(16, 1024 // n)), 1
        return ns1, max(1, min(16, 256 // n)), 4

    def scratch(self, cap: int):
        """Element counts of (scores, score statistics, partial outputs, counters)."""
        R = self.rows(cap)
        part = max(T * self.splits(T)[1] for T in range(1, R + 1)) if R < 4096 else 16 * R
        return (R * self.ks * self.hs, max(T * self.splits(T)[0] for T in range(1, R + 1)) * self.hs * 2, part * self.H * self.Dp,
                R * self.groups)


def talk_attention(plan: TalkPlan, q, kc, vc, talk, gate, out, scratch, block_tables, block_size: int, tok_seq, ctx_len, T: int,
                   V: int, scale: float, st: int):
    """Row-by-row attention with mixed heads (talk: TalkPlan.matrix); `gate`: a factor per output column, heads V columns apart."""
    p = plan
    ldg = gate.stride(0) if gate is not None else 0
    if gate is not None and gate.dtype != out.dtype:
        raise ValueError("talk_attention: a gate of the outputs' type")
    if not p.mfma:
        _check(lib().nls_talk_plain(q.data_ptr(), q.stride(0), kc.data_ptr(), vc.data_ptr(), block_tables.data_ptr(),
                                    block_tables.stride(0), block_size, tok_seq.data_ptr(), ctx_len.data_ptr(), T, p.H, p.G, p.Dp, V,
                                    scale, p.window, talk.data_ptr(), _p(gate), ldg, out.data_ptr(), out.stride(0),
                                    int(q.dtype == torch.float32), st), "nls_talk_plain")
        return
    sc, ss, po, cnt = scratch
    R = min(p.rows(T), sc.numel() // (p.ks * p.hs))
    for t0 in range(0, T, R):
        n = min(R, T - t0)
        ns1, ns, waves = p.splits(n)
        if (ss.numel() < n * ns1 * p.hs * 2 or cnt.numel() < n * p.groups or (ns > 1 and po.numel() < n * ns * p.H * p.Dp)):
            raise ValueError("talk_attention: workspace too small")
        _check(lib().nls_talk_decode(q.data_ptr(), q.stride(0), kc.data_ptr(), vc.data_ptr(), block_tables.data_ptr(),
                                     block_tables.stride(0), block_size, tok_seq.data_ptr(), ctx_len.data_ptr(), t0, n, p.H, p.G,
                                     p.Dp, V, scale, p.window, talk.data_ptr(), _p(gate), ldg, out.data_ptr(), out.stride(0),
                                     sc.data_ptr(), p.ks, ss.data_ptr(), po.data_ptr(), cnt.data_ptr(), ns1, ns, waves, st),
               "nls_talk_decode")


def talk_prefill(plan: TalkPlan, q, kc, vc, talk, gate, out, block_tables, block_size: int, blocks, nblocks: int, waves: int, V: int,
                 scale: float, st: int):
    """Attention with mixed heads of query blocks of up to 32 * waves tokens over their sequences' paged keys and values."""
    p = plan
    if not p.prefill or (gate is not None and gate.dtype != out.dtype):
        raise ValueError("talk_prefill: a shape of the row-by-row kernels, or a gate of another type")
    _check(lib().nls_talk_prefill(q.data_ptr(), q.stride(0), kc.data_ptr(), vc.data_ptr(), block_tables.data_ptr(),
                                  block_tables.stride(0), block_size, blocks.data_ptr(), nblocks, 2 * waves, p.H, p.G, p.Dp, V, scale, p.window, talk.data_ptr(), _p(gate),
                                  gate.stride(0) if gate is not None else 0, out.data_ptr(), out.stride(0), st), "nls_talk_prefill")
