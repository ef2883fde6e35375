"""Configuration of the config-driven decoder stacks: a folder with `config.json` and `model.safetensors`.

config.json names the design (`architecture`), the sizes of the model and, layer by layer, the mixer and the
feed-forward. What a design fixes for all of its models (where the norms sit, the norm's kind, activations, how the router
scores) is its `Design` entry here; a mechanism takes those constants as parameters."""
from __future__ import annotations

import json
import os
from dataclasses import dataclass, field
from typing import List, Optional


def default_ctx() -> int:
    """Context length of a stack model: the designs set no limit, the position and block tables are sized by this one."""
    return int(os.environ.get("NLS_STACK_CTX", "32768"))


@dataclass(frozen=True)
class Design:
    """What every model of a design has in common."""
    norm: str = "layer"                # layer: (x - mean) / sqrt(var + eps) * w; rms: x / rms(x) * w
    norm_one: bool = False             # the norm's weights are stored around zero: factor 1 + w
    norm_place: str = "output"         # output: x + norm(sublayer(x)), the sublayers read x itself
                                       # shared: h = norm(x), x + mixer(h) + feed-forward(h)
                                       # parallel: x + mixer(norm1(x)) + feed-forward(norm2(x))
                                       # sandwich: x + norm1b(mixer(norm1(x))), then the same with norm2, norm2b
    mixers: tuple = ()
    feed_forwards: tuple = ()
    rotary: str = "interleaved"        # pairs (2i, 2i + 1); halves: pairs (i, i + dims / 2)
    expert_act: str = "relu2"          # down(relu(up)^2), or silu_glu: down(silu(gate) * up)
    router_score: str = "sigmoid"      # or softmax, over all experts
    router_group: str = "top2"         # score of a group of experts: the sum of its two best, or max
    glu_act: str = "gelu_tanh"         # dense feed-forward: down(act(gate) * up), or clamped_swiglu: both clamped by the
                                       # config's limit, down(gate sigmoid(1.702 gate) (up + 1)); poly_norm: no gate,
                                       # down(a n(z) + b n(z^2) + c n(z^3) + e) of z = up, n an RMS norm over the ff values
    attn_qk_norm: str = "projection"   # attention: one RMS norm over all heads of the queries, one over the keys'; head: each
                                       # rotated head on its own, without weights; none
    attn_values: str = "keys"          # attention: the values are the projected keys, unnormed and unrotated; projection
    attn_gate: object = "head"         # attention: a sigmoid gate per head; column: per output column; None
    attn_talk: bool = False            # attention: the heads' softmax weights are mixed by a matrix [heads, heads]
    attn_sink: bool = False            # attention: the softmax's denominator holds one more, a score of 0 without a value
    tied_head: bool = False            # the logits are products with the (unscaled) embedding table
    positions: bool = False            # a learned vector per position is added to the embedding
    loop_entry: str = "product"        # looped layers, ahead of each pass: x = loop.in [x, embedding] + step; add: x + step


DESIGNS = {
    "Sekolorn": Design(mixers=("wkv", "latent_attention"), feed_forwards=("moe",)),
    "Kolodra": Design(norm="rms", norm_one=True, norm_place="shared", mixers=("parallel",), feed_forwards=("dense",)),
    "Bibapel": Design(norm="rms", norm_place="parallel", mixers=("channel_delta", "attention", "lightning"),
                      feed_forwards=("dense",), glu_act="clamped_swiglu", attn_qk_norm="none", attn_values="projection",
                      attn_gate=None, attn_sink=True, tied_head=True, positions=True),
    "Pimodra": Design(norm="rms", norm_place="sandwich", mixers=("attention",), feed_forwards=("dense", "moe"), rotary="halves",
                      expert_act="silu_glu", router_score="softmax", router_group="max", glu_act="poly_norm",
                      attn_qk_norm="head", attn_values="projection", attn_gate="column", attn_talk=True, tied_head=True,
                      loop_entry="add"),
}


@dataclass
class WkvConfig:
    heads: int
    dim: int
    kind, recurrent = "wkv", True


@dataclass
class LatentConfig:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    q_rank: int
    rot_base: float
    scale: float
    kv_from: Optional[int] = None
    kind, recurrent = "latent_attention", False


@dataclass
class RotScaling:
    """YaRN: wavelengths that turn at least `fast` times over the original length stay, those that turn at most `slow` times are
    stretched by `factor`, with a ramp between them; sine and cosine grow by 0.1 ln(factor) + 1."""
    factor: float
    original: float
    fast: float
    slow: float


@dataclass
class AttentionConfig:
    """Grouped-query softmax attention, optionally with partial rotary positions, or over a sliding window and the first
    tokens: position i sees j <= i if i - j < window or j < keep_first."""
    heads: int
    kv_heads: int
    dim: int                           # of queries and keys
    rot_dims: int
    rot_base: float
    scale: float
    vdim: int = 0                      # of values
    window: int = 0                    # 0: every earlier position is seen
    keep_first: int = 0
    rot_scaling: Optional[RotScaling] = None
    kind, recurrent = "attention", False


@dataclass
class GlaConfig:
    """Gated linear attention: a state [dim, vdim] per head, decayed per key channel by sigmoid(.)^(1 / tau)."""
    heads: int
    dim: int
    vdim: int
    tau: float
    kind, recurrent = "gla", True


@dataclass
class LightningConfig:
    """Linear attention with one constant decay per head, a state [dim, vdim] per head."""
    heads: int
    dim: int
    vdim: int
    decay: List[float]
    kind, recurrent = "lightning", True


@dataclass
class DeltaConfig:
    """Gated delta rule: a state [dim, vdim] per head, decayed per key channel, that each token corrects towards its value;
    queries, keys and values pass a causal convolution of `conv` taps. Queries and keys have kv_heads heads."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    kind, recurrent = "channel_delta", True


@dataclass
class ParallelConfig:
    """Two mixers on the same input, their outputs weighted and added."""
    left: AttentionConfig
    right: GlaConfig
    left_scale: float
    right_scale: float
    kind, recurrent = "parallel", True


@dataclass
class MoeConfig:
    experts: int
    top: int
    ff: int
    scale: float = 1.0
    groups: int = 1
    keep: int = 1
    shared_ff: int = 0                 # 0: no shared expert
    kind = "moe"


@dataclass
class DenseConfig:
    ff: int
    limit: float = 0.0                 # clamped_swiglu: bound of gate (above) and up (both sides)
    kind = "dense"
    experts = top = 0


@dataclass
class LayerConfig:
    mixer: object
    mlp: object = None                 # MoeConfig, DenseConfig or None
    weights_of: Optional[int] = None   # the layer whose tensors this one uses (resolved: never itself such a layer)


@dataclass
class BigramConfig:
    """A table row per pair of neighbouring tokens: (previous * mul_prev + current * mul_cur) mod buckets; the last row is that
    of a sequence's first token."""
    buckets: int
    mul_prev: int
    mul_cur: int


@dataclass
class LoopConfig:
    """Layers start .. stop - 1 run `times` times in a row with the same weights."""
    start: int
    stop: int
    times: int


@dataclass
class StackConfig:
    arch: str
    design: Design
    d_model: int
    vocab: int
    eps: float
    layers: List[LayerConfig] = field(default_factory=list)
    ctx: int = 32768
    embed_scale: float = 1.0
    softcap: float = 0.0               # logits: softcap * tanh(logits / softcap); 0: none
    bigram: Optional[BigramConfig] = None
    loop: Optional[LoopConfig] = None
    max_positions: int = 0             # rows of the learned positions (0: none)
    norm_groups: int = 1               # equal parts of the residual that the norms take each on its own

    @property
    def n_layer(self) -> int:
        return len(self.layers)

    @property
    def order(self) -> List[tuple]:
        """The layer runs of a forward pass: (layer, the loop's pass that starts with this run or None)."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, None) for i in range(n)]
        a, z = self.loop.start, self.loop.stop
        passes = [(i, t if i == a else None) for t in range(self.loop.times) for i in range(a, z)]
        return [(i, None) for i in range(a)] + passes + [(i, None) for i in range(z, n)]

    @property
    def n_expert(self) -> int:
        return max([L.mlp.experts for L in self.layers if L.mlp is not None], default=0)

    @property
    def n_expert_used(self) -> int:
        return max([L.mlp.top for L in self.layers if L.mlp is not None], default=0)

    @property
    def recurrent(self) -> bool:
        """Sequences carry state besides the paged cache: some layer's, or the previous token."""
        return self.bigram is not None or any(L.mixer.recurrent for L in self.layers)

    @classmethod
    def from_json(cls, cfg: dict, shape=None) -> "StackConfig":
        """`shape(name) -> tuple or None`: the checkpoint's tensor shapes, for sizes the config leaves to them."""
        arch = cfg.get("architecture")
        if arch not in DESIGNS:
            raise NotImplementedError(f"architecture {arch!r} not supported (supported: {sorted(DESIGNS)})")
        design = DESIGNS[arch]
        shape = shape or (lambda name: None)

        def size(d, key, name, axis=0, per=1):
            if key in d:
                return int(d[key])
            s = shape(name)
            if s is None:
                raise ValueError(f"config.json: {key!r} is missing and no tensor {name!r} gives it")
            return int(s[axis]) // per

        norm = cfg.get("norm") or {}
        out = cls(arch=arch, design=design, d_model=size(cfg, "width", "embed", 1), vocab=size(cfg, "vocab", "embed"),
                  eps=float(norm["eps"]), ctx=default_ctx(),
                  embed_scale=float((cfg.get("embedding") or {}).get("scale", 1.0)),
                  softcap=float(cfg.get("logit_softcap") or 0.0), norm_groups=int(norm.get("groups", 1)))
        if out.norm_groups < 1 or out.d_model % out.norm_groups or (out.norm_groups > 1 and design.norm != "rms"):
            raise ValueError(f"config.json: {out.norm_groups} norm groups of {out.d_model} columns")
        if design.positions:
            out.max_positions = size(cfg, "max_positions", "pos")
            out.ctx = min(out.ctx, out.max_positions)
        bg = (cfg.get("embedding") or {}).get("bigram")
        if bg is not None:
            rows = shape("bigram")
            out.bigram = BigramConfig(int(bg["buckets"]) if "buckets" in bg else int(rows[0]) - 1, int(bg["mul_prev"]),
                                      int(bg["mul_cur"]))
            if out.bigram.buckets < 1 or max(abs(out.bigram.mul_prev), abs(out.bigram.mul_cur)) >= 1 << 31:
                raise ValueError("config.json: embedding.bigram needs buckets >= 1 and 32-bit factors")
        if cfg.get("loop"):
            lp = out.loop = LoopConfig(*(int(cfg["loop"][k]) for k in ("start", "stop", "times")))
            if not 0 <= lp.start < lp.stop <= len(cfg["layers"]) or lp.times < 1:
                raise ValueError(f"config.json: loop {cfg['loop']} of {len(cfg['layers'])} layers")

        def wkv(i, m, p):
            u = shape(p + "u")
            return WkvConfig(int(m["heads"]) if "heads" in m else int(u[0]), int(m["dim"]) if "dim" in m else int(u[1]))

        def latent(i, m, p):
            H = int(m["heads"]) if "heads" in m else int(shape(p + "g")[0])
            rd = int(m["rot_dim"]) if "rot_dim" in m else int(m["rot"]["dims"])
            src = m.get("kv_from")
            mix = LatentConfig(
                heads=H, rot_dim=rd, dim=size(m, "dim", p + "uk", 0, H), vdim=size(m, "vdim", p + "uv", 0, H),
                kv_rank=size(m, "kv_rank", p + "uk", 1), q_rank=size(m, "q_rank", p + "dq"),
                rot_base=float(m["rot"]["base"]), scale=float(m["scale"]), kv_from=None if src is None else int(src))
            if rd % 2 or int(m["rot"].get("dims", rd)) != rd:
                raise ValueError(f"layer {i}: the rotation covers the whole rotated part: rot.dims = rot_dim, even")
            if mix.kv_from is not None:
                if not 0 <= mix.kv_from < i:
                    raise ValueError(f"layer {i}: kv_from {mix.kv_from} is not an earlier layer")
                o = out.layers[mix.kv_from].mixer
                if o.kind != "latent_attention" or o.kv_from is not None or (o.kv_rank, o.rot_dim, o.rot_base) != (
                        mix.kv_rank, mix.rot_dim, mix.rot_base):
                    raise ValueError(f"layer {i}: kv_from {mix.kv_from} has no matching latent cache of its own")
            return mix

        def attention(i, m, p):
            own = design.attn_values == "projection"
            H = size(m, "heads", p + "g") if design.attn_gate == "head" else \
                size(m, "heads", p + "talk") if design.attn_talk else int(m["heads"])
            D = size(m, "dim", p + "q", 0, H)
            G = size(m, "kv_heads", p + "k", 0, D)
            V = size(m, "vdim", p + "v", 0, G) if own else int(m.get("vdim", D))
            rot = m.get("rot") or {"dims": 0, "base": 1.0}
            rd = int(rot.get("dims", D))
            sc = rot.get("scaling")
            if sc is not None:
                sc = RotScaling(*(float(sc[k]) for k in ("factor", "original", "fast", "slow")))
                if min(sc.factor, sc.original, sc.fast, sc.slow) <= 0 or float(rot["base"]) <= 1:
                    raise ValueError(f"layer {i}: rotation scaling {rot['scaling']} at base {rot['base']}")
            mask = m.get("mask") or {}
            window, keep = int(mask.get("size") or 0), int(mask.get("keep_first") or 0)
            if H % G:
                raise ValueError(f"layer {i}: {H} query heads do not divide into {G} key heads")
            if not own and V != D:
                raise ValueError(f"layer {i}: the values are the keys: vdim {m['vdim']} must be dim {D}")
            if rd % 2 or not 0 <= rd <= D:
                raise ValueError(f"layer {i}: {rd} rotated dimensions of heads of {D}")
            if mask and (window < 1 or keep < 0):
                raise ValueError(f"layer {i}: attention mask {mask}")
            if design.attn_talk and (keep or design.attn_sink):
                raise NotImplementedError(f"layer {i}: mixed heads with kept first tokens or a sink")
            return AttentionConfig(heads=H, kv_heads=G, dim=D, rot_dims=rd, rot_base=float(rot["base"]), scale=float(m["scale"]),
                                   vdim=V, window=window, keep_first=keep, rot_scaling=sc)

        def gla(i, m, p):
            V = size(m, "vdim", p + "norm")
            H = size(m, "heads", p + "v", 0, V)
            return GlaConfig(heads=H, dim=size(m, "dim", p + "k", 0, H), vdim=V, tau=float(m["tau"]))

        def lightning(i, m, p):
            decay = [float(a) for a in m["decay"]]
            H = int(m.get("heads", len(decay)))
            if len(decay) != H or not all(0.0 <= a <= 1.0 for a in decay):
                raise ValueError(f"layer {i}: {H} heads need as many decays between 0 and 1")
            return LightningConfig(heads=H, dim=size(m, "dim", p + "k", 0, H), vdim=size(m, "vdim", p + "v", 0, H), decay=decay)

        def channel_delta(i, m, p):
            H, V = size(m, "heads", p + "b"), size(m, "vdim", p + "norm")
            D = size(m, "dim", p + "a2", 0, H)
            G = size(m, "kv_heads", p + "k", 0, D)
            if H % G:
                raise ValueError(f"layer {i}: {H} heads do not divide into {G} query and key heads")
            return DeltaConfig(heads=H, kv_heads=G, dim=D, vdim=V, conv=size(m, "conv", p + "q.conv", 1))

        def parallel(i, m, p):
            return ParallelConfig(left=attention(i, m["left"], p + "left."), right=gla(i, m["right"], p + "right."),
                                  left_scale=float(m["left_scale"]), right_scale=float(m["right_scale"]))

        def moe(i, f, p):
            r = f["router"]
            g = r.get("groups") or {}
            E = size(r, "experts", p + "router")
            mlp = MoeConfig(experts=E, top=int(r["top"]), ff=size(f.get("expert") or {}, "ff", p + "e0.up"),
                            scale=float(r.get("scale", 1.0)), groups=int(g.get("count", 1)),
                            keep=int(g.get("keep", g.get("count", 1))))
            if f.get("shared") is not None:
                mlp.shared_ff = size(f["shared"], "ff", p + "shared.up")
            if E % mlp.groups or not 1 <= mlp.keep <= mlp.groups or not 1 <= mlp.top <= mlp.keep * (E // mlp.groups):
                raise ValueError(f"layer {i}: {E} experts in {mlp.groups} groups, {mlp.keep} kept, cannot give "
                                 f"{mlp.top} experts")
            return mlp

        def dense(i, f, p):
            return DenseConfig(ff=size(f, "ff", p + "up"),
                               limit=float(f["limit"]) if design.glu_act == "clamped_swiglu" else 0.0)

        mixers = {"wkv": wkv, "latent_attention": latent, "parallel": parallel, "attention": attention,
                  "lightning": lightning, "channel_delta": channel_delta}
        feed_forwards = {"moe": moe, "dense": dense}
        owners = weight_owners(cfg["layers"])
        for i, L in enumerate(cfg["layers"]):
            t, p = L["type"], f"l{owners[i]}."
            if t not in design.mixers:
                raise NotImplementedError(f"{arch}: layer {i}: mixer {t!r} not supported {design.mixers}")
            layer = LayerConfig(mixers[t](i, L["mixer"], p + "mix."), weights_of=None if owners[i] == i else owners[i])
            f = L.get("mlp")
            if f is not None:
                kind = f.get("kind", design.feed_forwards[0])
                if kind not in design.feed_forwards:
                    raise NotImplementedError(f"{arch}: layer {i}: feed-forward {kind!r} not supported")
                layer.mlp = feed_forwards[kind](i, f, p + "mlp.")
            out.layers.append(layer)
        for i, L in enumerate(out.layers):
            o = out.layers[owners[i]]
            if L.mixer != o.mixer or L.mlp != o.mlp:
                raise ValueError(f"layer {i}: its entry is not that of layer {owners[i]}, whose weights it uses")
        return out

    @classmethod
    def from_dir(cls, path: str, shape=None) -> "StackConfig":
        with open(os.path.join(path, "config.json")) as f:
            return cls.from_json(json.load(f), shape)


def weight_owners(layers: List[dict]) -> List[int]:
    """The layer that holds each layer's tensors (`weights_of`, possibly over several layers)."""
    out = []
    for i in range(len(layers)):
        j, seen = i, {i}
        while layers[j].get("weights_of") is not None:
            j = int(layers[j]["weights_of"])
            if not 0 <= j < len(layers) or j in seen:
                raise ValueError(f"layer {i}: weights_of {j} names no layer with tensors")
            seen.add(j)
        out.append(j)
    return out


def is_stack_dir(path: str) -> bool:
    return os.path.isdir(path) and all(os.path.isfile(os.path.join(path, f)) for f in ("config.json", "model.safetensors"))
