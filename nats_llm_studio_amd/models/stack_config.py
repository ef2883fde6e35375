"""Configuration of the config-driven decoder stacks: a folder with `config.json` and `model.safetensors`.

config.json names the design (`architecture`), the sizes of the model and, layer by layer, the mixer and the
feed-forward. What a design fixes for all of its models (where the norms sit, the norm's kind, the expert activation,
how the router scores) is its `Design` entry here; a mechanism takes those constants as parameters."""
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
    norm: str = "layer"                # layer: (x - mean) / sqrt(var + eps) * w
    norm_place: str = "output"         # output: x + norm(sublayer(x)), the sublayers read x itself
    mixers: tuple = ()
    feed_forwards: tuple = ()
    rotary: str = "interleaved"        # pairs (2i, 2i + 1)
    expert_act: str = "relu2"
    router_score: str = "sigmoid"


DESIGNS = {
    "Sekolorn": Design(mixers=("wkv", "latent_attention"), feed_forwards=("moe",)),
}


@dataclass
class WkvConfig:
    heads: int
    dim: int
    kind = "wkv"


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
    kind = "latent_attention"


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
class LayerConfig:
    mixer: object
    mlp: Optional[MoeConfig] = None


@dataclass
class StackConfig:
    arch: str
    design: Design
    d_model: int
    vocab: int
    eps: float
    layers: List[LayerConfig] = field(default_factory=list)
    ctx: int = 32768

    @property
    def n_layer(self) -> int:
        return len(self.layers)

    @property
    def n_expert(self) -> int:
        return max([L.mlp.experts for L in self.layers if L.mlp is not None], default=0)

    @property
    def n_expert_used(self) -> int:
        return max([L.mlp.top for L in self.layers if L.mlp is not None], default=0)

    @property
    def recurrent(self) -> bool:
        """Some layer carries per-sequence state besides the paged cache."""
        return any(L.mixer.kind == "wkv" for L in self.layers)

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
                  eps=float(norm["eps"]), ctx=default_ctx())
        for i, L in enumerate(cfg["layers"]):
            t, m, p = L["type"], L["mixer"], f"l{i}."
            if t not in design.mixers:
                raise NotImplementedError(f"{arch}: layer {i}: mixer {t!r} not supported {design.mixers}")
            if t == "wkv":
                u = shape(p + "mix.u")
                mix = WkvConfig(int(m["heads"]) if "heads" in m else int(u[0]),
                                int(m["dim"]) if "dim" in m else int(u[1]))
            else:
                H = int(m["heads"]) if "heads" in m else int(shape(p + "mix.g")[0])
                rd = int(m["rot_dim"]) if "rot_dim" in m else int(m["rot"]["dims"])
                src = m.get("kv_from")
                mix = LatentConfig(
                    heads=H, rot_dim=rd, dim=size(m, "dim", p + "mix.uk", 0, H), vdim=size(m, "vdim", p + "mix.uv", 0, H),
                    kv_rank=size(m, "kv_rank", p + "mix.uk", 1), q_rank=size(m, "q_rank", p + "mix.dq"),
                    rot_base=float(m["rot"]["base"]), scale=float(m["scale"]), kv_from=None if src is None else int(src))
                if rd % 2 or int(m["rot"].get("dims", rd)) != rd:
                    raise ValueError(f"layer {i}: the rotation covers the whole rotated part: rot.dims = rot_dim, even")
                if mix.kv_from is not None:
                    if not 0 <= mix.kv_from < i:
                        raise ValueError(f"layer {i}: kv_from {mix.kv_from} is not an earlier layer")
                    o = out.layers[mix.kv_from].mixer
                    if o.kind != t or o.kv_from is not None or (o.kv_rank, o.rot_dim, o.rot_base) != (
                            mix.kv_rank, mix.rot_dim, mix.rot_base):
                        raise ValueError(f"layer {i}: kv_from {mix.kv_from} has no matching latent cache of its own")
            mlp = None
            if L.get("mlp") is not None:
                f = L["mlp"]
                if f.get("kind", "moe") not in design.feed_forwards:
                    raise NotImplementedError(f"{arch}: layer {i}: feed-forward {f.get('kind')!r} not supported")
                r = f["router"]
                g = r.get("groups") or {}
                E = size(r, "experts", p + "mlp.router")
                mlp = MoeConfig(experts=E, top=int(r["top"]), ff=size(f.get("expert") or {}, "ff", p + "mlp.e0.up"),
                                scale=float(r.get("scale", 1.0)), groups=int(g.get("count", 1)),
                                keep=int(g.get("keep", g.get("count", 1))))
                if f.get("shared") is not None:
                    mlp.shared_ff = size(f["shared"], "ff", p + "mlp.shared.up")
                if E % mlp.groups or not 1 <= mlp.keep <= mlp.groups or not 1 <= mlp.top <= mlp.keep * (E // mlp.groups):
                    raise ValueError(f"layer {i}: {E} experts in {mlp.groups} groups, {mlp.keep} kept, cannot give "
                                     f"{mlp.top} experts")
            out.layers.append(LayerConfig(mix, mlp))
        return out

    @classmethod
    def from_dir(cls, path: str, shape=None) -> "StackConfig":
        with open(os.path.join(path, "config.json")) as f:
            return cls.from_json(json.load(f), shape)


def is_stack_dir(path: str) -> bool:
    return os.path.isdir(path) and all(os.path.isfile(os.path.join(path, f)) for f in ("config.json", "model.safetensors"))
