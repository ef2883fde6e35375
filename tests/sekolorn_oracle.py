"""Plain, slow implementation of the Sekolorn design (CPU, one sequence at a time, one function per mechanism).

The correctness oracle of the Sekolorn tests: float64 by default, token loops where the mechanism is a recurrence,
no caches, no batching, nothing shared with the product code. `weights` maps a tensor name to a torch tensor."""
from __future__ import annotations

import math

import torch


def layer_norm(x, w, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def rms_norm(x, w, eps):
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if w is None else y * w


def rotate(x, positions, base, dims):
    """Interleaved rotary embedding on the first `dims` of the last axis; x [n, ..., D], positions [n]."""
    out = x.clone()
    for i in range(dims // 2):
        a = positions.double() * float(base) ** (-2.0 * i / dims)
        c, s = torch.cos(a).to(x.dtype), torch.sin(a).to(x.dtype)
        while c.dim() < x.dim() - 1:
            c, s = c.unsqueeze(-1), s.unsqueeze(-1)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def token_shift(h, prev):
    """The previous token's row of every row of h; `prev` is the row before the first (None: zeros)."""
    first = torch.zeros_like(h[:1]) if prev is None else prev[None]
    return torch.cat([first, h[:-1]], 0)


def wkv_scan(r, k, v, w, u, state=None):
    """r, k, v, w: [n, heads, dim]; u [heads, dim]. Returns o [n, heads, dim] and the state [heads, dim, dim]."""
    n, H, D = r.shape
    S = torch.zeros(H, D, D, dtype=r.dtype) if state is None else state.clone()
    out = []
    for t in range(n):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out.append(((S + u[:, :, None] * kv) * r[t][:, :, None]).sum(1))
        S = w[t][:, :, None] * S + kv
    return torch.stack(out), S


def wkv_mixer(h, W, p, mix, eps, state=None):
    """state: None, or (previous token's h, S). Returns the mixer's output and the new state."""
    H, D = mix["heads"], mix["dim"]
    hp = token_shift(h, None if state is None else state[0])
    m = {s: h + (hp - h) * W[p + "mu." + s] for s in "rkvgw"}
    r, k, v = (((m[s] @ W[p + s].T).view(-1, H, D)) for s in "rkv")
    z = m["g"] @ W[p + "g"].T
    gate = z / (1 + torch.exp(-z))
    w = torch.exp(-torch.exp(torch.tanh(m["w"] @ W[p + "w1"].T) @ W[p + "w2"].T + W[p + "w0"])).view(-1, H, D)
    o, S = wkv_scan(r, k, v, w, W[p + "u"].view(H, D), None if state is None else state[1])
    o = rms_norm(o, None, eps).reshape(h.shape[0], H * D) * W[p + "norm"] * gate
    return o @ W[p + "o"].T, (h[-1], S)


def latent_rows(h, W, p, mix, positions, eps):
    """What a latent-attention layer caches per token: the normed latent c and the rotated shared key part."""
    z = h @ W[p + "dkv"].T
    R = mix["kv_rank"]
    kr = rotate(z[:, R:], positions, mix["rot"]["base"], mix["rot_dim"])
    return rms_norm(z[:, :R], W[p + "dkv.norm"], eps), kr


def latent_mixer(h, W, p, mix, positions, eps, c, kr):
    """c, kr: the rows of every token up to the last position of h (positions 0..)."""
    H, D, RD, VD = mix["heads"], mix["dim"], mix["rot_dim"], mix["vdim"]
    cq = rms_norm(h @ W[p + "dq"].T, W[p + "dq.norm"], eps)
    q = (cq @ W[p + "uq"].T).view(-1, H, D + RD)
    qr = rotate(q[..., D:], positions, mix["rot"]["base"], RD)
    k = (c @ W[p + "uk"].T).view(-1, H, D)
    v = (c @ W[p + "uv"].T).view(-1, H, VD)
    s = (torch.matmul(q[..., :D].transpose(0, 1), k.permute(1, 2, 0))
         + torch.matmul(qr.transpose(0, 1), kr.T)) * mix["scale"]
    keys = torch.arange(c.shape[0])
    s = s.masked_fill(keys[None, None, :] > positions[None, :, None], -math.inf)
    o = torch.matmul(torch.softmax(s, -1), v.transpose(0, 1)).transpose(0, 1)      # [n, H, VD]
    gate = 1 / (1 + torch.exp(-(h @ W[p + "g"].T)))
    return (o * gate[:, :, None]).reshape(h.shape[0], H * VD) @ W[p + "o"].T


def route(z, top, scale, groups, keep):
    """Router logits of ONE token -> [(expert, weight)]."""
    s = 1 / (1 + torch.exp(-z))
    E = s.shape[0]
    per = E // groups
    gs = [sum(sorted(s[g * per:(g + 1) * per].tolist(), reverse=True)[:2]) for g in range(groups)]
    ok = set(sorted(range(groups), key=lambda g: (-gs[g], g))[:keep])
    cand = [e for e in range(E) if e // per in ok]
    best = sorted(cand, key=lambda e: (-float(s[e]), e))[:top]
    return [(e, s[e] * scale) for e in best]


def expert(h, up, down):
    return torch.relu(h @ up.T) ** 2 @ down.T


def moe(h, W, p, mlp):
    r = mlp["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    z = h @ W[p + "router"].T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in route(z[t], r["top"], r["scale"], g["count"], g["keep"]):
            out[t] += w * expert(h[t], W[f"{p}e{e}.up"], W[f"{p}e{e}.down"])
    if mlp.get("shared"):
        out = out + expert(h, W[p + "shared.up"], W[p + "shared.down"])
    return out


def forward(cfg, weights, tokens, dtype=torch.float64, layers=None):
    """Logits [n, vocab] of a whole sequence; `layers` (a list) receives the residual after every layer."""
    W = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    pos = torch.arange(len(tokens))
    x = W["embed"][torch.tensor(tokens)]
    rows = {}
    for i, L in enumerate(cfg["layers"]):
        p, mix = f"l{i}.", L["mixer"]
        if L["type"] == "wkv":
            y, _ = wkv_mixer(x, W, p + "mix.", mix, eps)
        else:
            if "kv_from" in mix:
                c, kr = rows[mix["kv_from"]]
            else:
                c, kr = rows[i] = latent_rows(x, W, p + "mix.", mix, pos, eps)
            y = latent_mixer(x, W, p + "mix.", mix, pos, eps, c, kr)
        x = x + layer_norm(y, W[p + "norm1"], eps)
        if L.get("mlp"):
            x = x + layer_norm(moe(x, W, p + "mlp.", L["mlp"]), W[p + "norm2"], eps)
        if layers is not None:
            layers.append(x.clone())
    return layer_norm(x, W["final.norm"], eps) @ W["head"].T
