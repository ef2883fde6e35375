"""Plain, slow implementation of the Bibapel design (CPU, one sequence at a time, one function per mechanism).

The correctness oracle of the Bibapel tests: float64 by default, token loops where the mechanism is a recurrence, no
caches, no batching, nothing shared with the product code. `weights` maps a tensor name to a torch tensor."""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    """x over its root mean square (last axis)."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, w, eps):
    return rms(x, eps) * w


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-torch.abs(z)))


# ---- embedding

def bigram_row(prev, cur, b):
    """Row of the pair table; prev None: the sequence's first token."""
    if prev is None:
        return b["buckets"]
    return (int(prev) * b["mul_prev"] + int(cur) * b["mul_cur"]) % b["buckets"]


def embed(cfg, W, tokens, prev=None, first=0):
    """Rows of `tokens` at positions first, first + 1, ..; `prev` the token ahead of them."""
    out = []
    e = cfg["embedding"]
    for i, t in enumerate(tokens):
        x = W["embed"][t] * e["scale"]
        if e.get("bigram"):
            x = x + W["bigram"][bigram_row(prev, t, e["bigram"])]
        out.append(x + W["pos"][first + i])
        prev = t
    return torch.stack(out)


# ---- attention

def visible(i, j, mask):
    """Whether position i sees position j (tensors of positions)."""
    if not mask:
        return j <= i
    return (j <= i) & ((i - j < mask["size"]) | (j < mask["keep_first"]))


def attend(q, k, v, positions, scale, mask):
    """q [n, H, D] at `positions` over k [N, G, D], v [N, G, V] of positions 0 .. N - 1; one is added to the softmax's
    denominator."""
    H, G = q.shape[1], k.shape[1]
    out = torch.zeros(q.shape[0], H, v.shape[2], dtype=q.dtype)
    see = visible(positions[:, None], torch.arange(k.shape[0])[None, :], mask)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T * scale).masked_fill(~see, -math.inf)
        m = torch.clamp(s.max(-1, keepdim=True).values, min=0.0)
        out[:, h] = sink_weights(torch.exp(s - m), torch.exp(-m)) @ v[:, g]
    return out


def sink_weights(e, one):
    """Softmax weights with one more in the denominator; both scaled by the same factor."""
    return e / (one + e.sum(-1, keepdim=True))


def attention_mixer(h, W, p, m, positions, eps, before=None):
    """`before`: the keys and values of the tokens ahead of h's first. Returns the output and all keys and values."""
    H, G = m["heads"], m["kv_heads"]
    q = (h @ W[p + "q"].T).reshape(-1, H, m["dim"])
    k = (h @ W[p + "k"].T).reshape(-1, G, m["dim"])
    v = (h @ W[p + "v"].T).reshape(-1, G, m["vdim"])
    if before is not None:
        k, v = torch.cat([before[0], k]), torch.cat([before[1], v])
    o = attend(q, k, v, positions, m["scale"], m.get("mask"))
    return o.reshape(h.shape[0], -1) @ W[p + "o"].T, (k, v)


# ---- linear attention with one decay per head

def lightning_scan(q, k, v, decay, state=None):
    """q, k [n, heads, dim], v [n, heads, vdim], decay [heads]; the state is updated, then read."""
    S = torch.zeros(q.shape[1], q.shape[2], v.shape[2], dtype=q.dtype) if state is None else state.clone()
    out = []
    for t in range(q.shape[0]):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def lightning_mixer(h, W, p, m, positions, eps, before=None):
    H = m["heads"]
    q, k, v = (silu(h @ W[p + n].T).reshape(h.shape[0], H, -1) for n in "qkv")
    o, S = lightning_scan(q, k, v, torch.tensor(m["decay"], dtype=h.dtype), before)
    o = norm(o.reshape(h.shape[0], -1), W[p + "norm"], eps) * sigmoid(h @ W[p + "g"].T)
    return o @ W[p + "o"].T, S


# ---- delta rule with one decay per key channel

def causal_conv(x, w, before=None):
    """x [n, channels], w [channels, taps] (last: the current token); `before`: the taps - 1 inputs ahead (zeros at the
    start). Returns the outputs and the last taps - 1 inputs."""
    taps = w.shape[1]
    if before is None:
        before = torch.zeros(taps - 1, x.shape[1], dtype=x.dtype)
    full = torch.cat([before, x])
    out = torch.stack([sum(full[t + j] * w[:, j] for j in range(taps)) for t in range(x.shape[0])])
    return out, full[full.shape[0] - (taps - 1):]


def delta_decay(h, W, p, m):
    """[n, heads, dim]"""
    z = (h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "dt_bias"]
    z = softplus(z).reshape(-1, m["heads"], m["dim"])
    return torch.exp(-torch.exp(W[p + "A_log"])[None, :, None] * z)


def delta_scan(q, k, v, g, beta, state=None):
    """q, k, g [n, heads, dim], v [n, heads, vdim], beta [n, heads]: decay, correct the state's answer to k towards v, read."""
    S = torch.zeros(q.shape[1], q.shape[2], v.shape[2], dtype=q.dtype) if state is None else state.clone()
    out = []
    for t in range(q.shape[0]):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def delta_mixer(h, W, p, m, positions, eps, before=None):
    H, G, D, n = m["heads"], m["kv_heads"], m["dim"], h.shape[0]
    S, tails = (None, (None, None, None)) if before is None else before
    acts, ends = [], []
    for name, tail in zip("qkv", tails):
        y, e = causal_conv(h @ W[p + name].T, W[p + name + ".conv"], tail)
        acts.append(silu(y))
        ends.append(e)
    q, k, v = acts
    of = torch.arange(H) // (H // G)
    q = (unit(q.reshape(n, G, D)) * D ** -0.5)[:, of]
    k = unit(k.reshape(n, G, D))[:, of]
    beta = sigmoid(h @ W[p + "b"].T)
    o, S = delta_scan(q, k, v.reshape(n, H, -1), delta_decay(h, W, p, m), beta, S)
    o = norm(o, W[p + "norm"], eps).reshape(n, -1) * sigmoid((h @ W[p + "g1"].T) @ W[p + "g2"].T)
    return o @ W[p + "o"].T, (S, tuple(ends))


MIXERS = {"attention": "attention_mixer", "lightning": "lightning_mixer", "channel_delta": "delta_mixer"}


# ---- feed-forward, layers, passes

def dense_ff(h, W, p, limit):
    g = torch.clamp(h @ W[p + "gate"].T, max=limit)
    u = torch.clamp(h @ W[p + "up"].T, min=-limit, max=limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ W[p + "down"].T


def layer(x, W, p, L, positions, eps, before=None):
    y, after = globals()[MIXERS[L["type"]]](norm(x, W[p + "norm1"], eps), W, p + "mix.", L["mixer"], positions, eps, before)
    if L.get("mlp"):
        y = y + dense_ff(norm(x, W[p + "norm2"], eps), W, p + "mlp.", L["mlp"]["limit"])
    return x + y, after


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


def enter_pass(x, x0, W, t):
    return torch.cat([x, x0], -1) @ W["loop.in"].T + W["loop.step"][t]


def forward(cfg, weights, tokens, dtype=torch.float64, layers=None):
    """Logits [n, vocab] of a whole sequence; `layers` (a list) receives the residual after every layer run."""
    W = {k: v.to(dtype) if v.is_floating_point() else v for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    pos = torch.arange(len(tokens))
    x = x0 = embed(cfg, W, tokens)
    for i, t in order(cfg):
        if t is not None:
            x = enter_pass(x, x0, W, t)
        x, _ = layer(x, W, f"l{i}.", cfg["layers"][i], pos, eps)
        if layers is not None:
            layers.append(x.clone())
    return norm(x, W["final.norm"], eps) @ W["embed"].T
