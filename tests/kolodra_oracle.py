"""Plain, slow implementation of the Kolodra design (CPU, one sequence at a time, one function per mechanism).

The correctness oracle of the Kolodra tests: float64 by default, token loops where the mechanism is a recurrence, no
caches, no batching, nothing shared with the product code. `weights` maps a tensor name to a torch tensor."""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    """x over its root mean square (last axis)."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_one_plus(x, w, eps):
    return rms(x, eps) * (1.0 + w)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z * z * z)))


def rotate(x, positions, base, dims):
    """Rotary positions on the first `dims` of the last axis, neighbours paired; x [n, heads, D], positions [n]."""
    out = x.clone()
    for i in range(dims // 2):
        a = positions.double() * float(base) ** (-2.0 * i / dims)
        c, s = torch.cos(a).to(x.dtype)[:, None], torch.sin(a).to(x.dtype)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def attention_rows(h, W, p, m, positions, eps):
    """Queries [n, H, D], keys [n, G, D] and values [n, G, D] of the tokens: the queries and keys normed over their whole
    projection and rotated; a value is its key ahead of both."""
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    q, k = h @ W[p + "q"].T, h @ W[p + "k"].T
    v = k.reshape(-1, G, D)
    q = (rms(q, eps) * W[p + "q.norm"]).reshape(-1, H, D)
    k = (rms(k, eps) * W[p + "k.norm"]).reshape(-1, G, D)
    r = m["rot"]
    return rotate(q, positions, r["base"], r["dims"]), rotate(k, positions, r["base"], r["dims"]), v


def attend(q, k, v, positions, scale):
    """Causal softmax attention: q [n, H, D] at `positions` over k, v [N, G, D] of positions 0 .. N - 1."""
    H, G = q.shape[1], k.shape[1]
    out = torch.zeros(q.shape[0], H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        s = q[:, h] @ k[:, g].T * scale
        s = s.masked_fill(torch.arange(k.shape[0])[None, :] > positions[:, None], -math.inf)
        out[:, h] = torch.softmax(s, -1) @ v[:, g]
    return out


def attention_mixer(h, W, p, m, positions, eps, before=None):
    """`before`: the keys and values of the tokens ahead of h's first. Returns the output and all keys and values."""
    q, k, v = attention_rows(h, W, p, m, positions, eps)
    if before is not None:
        k, v = torch.cat([before[0], k]), torch.cat([before[1], v])
    o = attend(q, k, v, positions, m["scale"])
    o = o * sigmoid(h @ W[p + "g"].T)[:, :, None]
    return o.reshape(h.shape[0], -1) @ W[p + "o"].T, (k, v)


def decay(h, W, p, m):
    """alpha [n, heads, dim]."""
    z = (h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "a2.b"]
    return (sigmoid(z) ** (1.0 / m["tau"])).reshape(-1, m["heads"], m["dim"])


def gla_scan(q, k, v, a, state=None):
    """q, k, a [n, heads, dim], v [n, heads, vdim]; the state [heads, dim, vdim] is updated, then read."""
    S = torch.zeros(q.shape[1], q.shape[2], v.shape[2], dtype=q.dtype) if state is None else state.clone()
    out = []
    for t in range(q.shape[0]):
        S = a[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def gla_mixer(h, W, p, m, eps, state=None):
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q = (h @ W[p + "q"].T * D ** -0.5).reshape(-1, H, D)
    k = (h @ W[p + "k"].T).reshape(-1, H, D)
    v = (h @ W[p + "v"].T).reshape(-1, H, V)
    o, S = gla_scan(q, k, v, decay(h, W, p, m), state)
    o = (rms(o, eps) * W[p + "norm"]).reshape(h.shape[0], H * V)
    return (o * silu(h @ W[p + "g"].T)) @ W[p + "o"].T, S


def parallel_mixer(h, W, p, m, positions, eps, before=None):
    kv, S = (None, None) if before is None else before
    left, kv = attention_mixer(h, W, p + "left.", m["left"], positions, eps, kv)
    right, S = gla_mixer(h, W, p + "right.", m["right"], eps, S)
    return m["left_scale"] * left + m["right_scale"] * right, (kv, S)


def dense_ff(h, W, p):
    return (gelu_tanh(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def softcap(z, cap):
    return cap * torch.tanh(z / cap)


def owner(cfg, i):
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def forward(cfg, weights, tokens, dtype=torch.float64, layers=None):
    """Logits [n, vocab] of a whole sequence; `layers` (a list) receives the residual after every layer."""
    W = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    pos = torch.arange(len(tokens))
    x = W["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{owner(cfg, i)}."
        h = norm_one_plus(x, W[p + "norm1"], eps)
        y, _ = parallel_mixer(h, W, p + "mix.", L["mixer"], pos, eps)
        if L.get("mlp"):
            y = y + dense_ff(h, W, p + "mlp.")
        x = x + y
        if layers is not None:
            layers.append(x.clone())
    return softcap(norm_one_plus(x, W["final.norm"], eps) @ W["head"].T, cfg["logit_softcap"])
