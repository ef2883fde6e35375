"""Plain, slow implementation of the Pimodra design (CPU, one sequence at a time, one function per mechanism).

The correctness oracle of the Pimodra tests: float64 by default, no caches beyond the keys and values handed on, no batching,
nothing shared with the product code. `weights` maps a tensor name to a torch tensor."""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    """x over its root mean square (last axis)."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, w, eps, groups):
    """Each of `groups` consecutive parts of the last axis over its own root mean square, the whole times w."""
    return rms(x.reshape(*x.shape[:-1], groups, -1), eps).reshape(x.shape) * w


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


# ---- rotary positions

def frequencies(rot):
    """Angle per position of each rotated pair, and the factor of its sine and cosine: long wavelengths are stretched by the
    scaling's factor, short ones stay, a ramp over the pair's number between them."""
    dims, base, sc = rot["dims"], rot["base"], rot.get("scaling")
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if sc is None:
        return f, 1.0

    def turns(t):                               # the (real) pair number that makes t turns over the original length
        return dims * math.log(sc["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(turns(sc["fast"])), 0), min(math.ceil(turns(sc["slow"])), dims - 1)
    out = []
    for i, v in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(v / sc["factor"] * ramp + v * (1.0 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, positions, rot):
    """x [n, heads, dim]: column i of the first half of the rotated dims turns with column i of the second half."""
    f, gain = frequencies(rot)
    half = rot["dims"] // 2
    out = x.clone()
    for i in range(half):
        a = positions.to(x.dtype) * f[i]
        c, s = (torch.cos(a) * gain)[:, None], (torch.sin(a) * gain)[:, None]
        u, v = x[:, :, i], x[:, :, i + half]
        out[:, :, i] = u * c - v * s
        out[:, :, i + half] = v * c + u * s
    return out


# ---- attention

def visible(i, j, mask):
    """Whether position i sees position j (tensors of positions)."""
    see = j <= i
    return see & (i - j < mask["size"]) if mask else see


def mix_heads(w, talk):
    """w [heads, n, keys]: head h's weights become the sum over heads g of talk[h, g] w[g]."""
    out = torch.zeros_like(w)
    for h in range(w.shape[0]):
        for g in range(w.shape[0]):
            out[h] += talk[h, g] * w[g]
    return out


def attend(q, k, v, positions, scale, mask, talk):
    """q [n, H, D] at `positions` over k [N, G, D], v [N, G, V] of positions 0 .. N - 1."""
    H, G = q.shape[1], k.shape[1]
    see = visible(positions[:, None], torch.arange(k.shape[0])[None, :], mask)
    w = []
    for h in range(H):
        s = (q[:, h] @ k[:, h // (H // G)].T * scale).masked_fill(~see, -math.inf)
        e = torch.exp(s - s.max(-1, keepdim=True).values)
        w.append(e / e.sum(-1, keepdim=True))
    w = mix_heads(torch.stack(w), talk)
    return torch.stack([w[h] @ v[:, h // (H // G)] for h in range(H)], 1)


def output_gate(o, h, wg):
    return o * sigmoid(h @ wg.T)


def attention_mixer(h, W, p, m, positions, eps, before=None):
    """`before`: the keys and values of the tokens ahead of h's first. Returns the output and all keys and values."""
    H, G, n = m["heads"], m["kv_heads"], h.shape[0]
    q = (h @ W[p + "q"].T).reshape(n, H, m["dim"])
    k = (h @ W[p + "k"].T).reshape(n, G, m["dim"])
    v = (h @ W[p + "v"].T).reshape(n, G, m["vdim"])
    if m.get("rot"):
        q, k = rotate(q, positions, m["rot"]), rotate(k, positions, m["rot"])
    q, k = rms(q, eps), rms(k, eps)
    if before is not None:
        k, v = torch.cat([before[0], k]), torch.cat([before[1], v])
    o = attend(q, k, v, positions, m["scale"], m.get("mask"), W[p + "talk"])
    return output_gate(o.reshape(n, -1), h, W[p + "g"]) @ W[p + "o"].T, (k, v)


# ---- feed-forwards

def poly_norm(z, act, eps):
    a, b, c, e = act
    return a * rms(z, eps) + b * rms(z * z, eps) + c * rms(z * z * z, eps) + e


def dense_ff(h, W, p, f, eps):
    return poly_norm(h @ W[p + "up"].T, W[p + "act"], eps) @ W[p + "down"].T


def router_scores(z):
    e = torch.exp(z - z.max())
    return e / e.sum()


def group_score(s):
    return s.max()


def choose(s, router):
    """Experts of one token's scores, best first."""
    g = router.get("groups") or {"count": 1, "keep": 1}
    per = len(s) // g["count"]
    score = [float(group_score(s[i * per:(i + 1) * per])) for i in range(g["count"])]
    kept = sorted(range(g["count"]), key=lambda i: -score[i])[:g["keep"]]
    return sorted((e for i in kept for e in range(i * per, (i + 1) * per)), key=lambda e: -float(s[e]))[:router["top"]]


def expert(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def expert_weights(s, chosen):
    return s[chosen]


def moe_ff(h, W, p, f, eps):
    out = []
    for x in h:
        s = router_scores(W[p + "router"] @ x)
        chosen = choose(s, f["router"])
        out.append(sum(w * expert(x[None], W, f"{p}e{e}.")[0] for w, e in zip(expert_weights(s, chosen), chosen)))
    return torch.stack(out)


FEED_FORWARDS = {"dense": "dense_ff", "moe": "moe_ff"}


# ---- layers, passes

def layer(x, W, p, L, positions, nrm, before=None):
    """nrm: the config's norm (eps, groups)."""
    eps, groups = nrm["eps"], nrm["groups"]
    y, after = attention_mixer(norm(x, W[p + "norm1"], eps, groups), W, p + "mix.", L["mixer"], positions, eps, before)
    x = x + norm(y, W[p + "norm1b"], eps, groups)
    if L.get("mlp"):
        ff = globals()[FEED_FORWARDS[L["mlp"]["kind"]]]
        y = ff(norm(x, W[p + "norm2"], eps, groups), W, p + "mlp.", L["mlp"], eps)
        x = x + norm(y, W[p + "norm2b"], eps, groups)
    return x, after


def order(cfg):
    """[(layer, pass that starts here or None)]"""
    loop, n = cfg.get("loop"), len(cfg["layers"])
    if not loop:
        return [(i, None) for i in range(n)]
    a, z = loop["start"], loop["stop"]
    out = [(i, None) for i in range(a)]
    for t in range(loop["times"]):
        out += [(i, t if i == a else None) for i in range(a, z)]
    return out + [(i, None) for i in range(z, n)]


def enter_pass(x, W, t):
    return x + W["loop.step"][t]


def forward(cfg, weights, tokens, dtype=torch.float64, layers=None):
    """Logits [n, vocab] of a whole sequence; `layers` (a list) receives the residual after every layer run."""
    W = {k: v.to(dtype) if v.is_floating_point() else v for k, v in weights.items()}
    nrm = dict(cfg["norm"], groups=cfg["norm"].get("groups", 1))
    pos = torch.arange(len(tokens))
    x = W["embed"][torch.as_tensor(tokens)]
    for i, t in order(cfg):
        if t is not None:
            x = enter_pass(x, W, t)
        x, _ = layer(x, W, f"l{i}.", cfg["layers"][i], pos, nrm)
        if layers is not None:
            layers.append(x.clone())
    return norm(x, W["final.norm"], nrm["eps"], nrm["groups"]) @ W["embed"].T
