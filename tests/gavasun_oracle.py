"""Plain, slow float64 implementation of the Gavasun design, one function per mechanism.

It is the yardstick of the Gavasun tests and shares no code with the engine: it takes a config dict (the layout of
config.json) and a dict name -> torch tensor, runs one whole sequence at a time and keeps no cache (attention looks at
the whole prefix, the recurrence is walked token by token from a zero state, convolutions see zeros before the first
token).

Notation: n tokens, width E. Linear weights are [out, in]; y = x @ W.T. A layer is x <- x + mixer(N1(x)), then
x <- x + ff(N2(x)), where N(x) = x / rms(x) * (1 + w).
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def centred_norm(x, w, eps):
    """RMS norm whose stored weight is the distance from one."""
    return unit_rms(x, eps) * (1.0 + w)


def silu(z):
    return z * torch.sigmoid(z)


def gelu(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + torch.clamp(z, min=0.0)


def causal_conv(x, w):
    """x [n, C], w [C, taps]: sum_j w[:, j] x_(t - taps + 1 + j); zeros before the sequence's start."""
    n, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x)
    for t in range(n):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                out[t] += w[:, j] * x[s]
    return out


# --------------------------------------------------------------------------------------------- positions
def frequencies(rot):
    """(frequencies, amplitude): f_i = base^(-2i/dims); with YaRN scaling, dimensions that turn often keep theirs,
    slow ones are divided by the factor, a linear ramp over the index between; cos and sin grow by 1 + 0.1 ln(factor)."""
    dims, base, sc = rot["dims"], rot["base"], rot.get("scaling")
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not sc:
        return f, 1.0

    def at(turns):
        return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(at(sc["fast"])), 0)
    hi = min(math.ceil(at(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * ramp + fi * (1.0 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, rot, adjacent):
    """x [n, heads, D], row = position. Pairs (2i, 2i + 1) if `adjacent`, else (i, i + dims / 2)."""
    if not rot or not rot.get("dims"):
        return x
    f, amp = frequencies(rot)
    half = len(f)
    out = x.clone()
    for p in range(x.shape[0]):
        for i in range(half):
            a = p * f[i]
            c, s = amp * math.cos(a), amp * math.sin(a)
            iu, iv = (2 * i, 2 * i + 1) if adjacent else (i, i + half)
            u, v = x[p, :, iu], x[p, :, iv]
            out[p, :, iu] = u * c - v * s
            out[p, :, iv] = v * c + u * s
    return out


def in_window(n, size):
    """Position i sees j with 0 <= i - j < size."""
    d = torch.arange(n)[:, None] - torch.arange(n)[None, :]
    return (d >= 0) & (d < size)


def in_chunk(n, size):
    """Position i sees j <= i of the same block of `size` positions, blocks counted from position 0."""
    i = torch.arange(n)
    return (i[None, :] <= i[:, None]) & (i[None, :] // size == i[:, None] // size)


def visible(n, rule, m):
    """Mask of one layer; without a size every earlier position is seen."""
    size = (m.get("mask") or {}).get("size")
    return rule(n, size) if size else in_window(n, n)


# --------------------------------------------------------------------------------------------- mixers
def gated_delta(h, W, m, eps):
    """Delta rule with one decay per head: the state forgets, then what it would answer to the new key is taken off the
    new value (times beta) before it is written, then it is read."""
    n, H, G, D, Dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = silu(causal_conv(h @ W["q"].T, W["q.conv"])).view(n, G, D)
    k = silu(causal_conv(h @ W["k"].T, W["k.conv"])).view(n, G, D)
    v = silu(causal_conv(h @ W["v"].T, W["v.conv"])).view(n, H, Dv)
    q = q / torch.sqrt((q * q).sum(-1, keepdim=True) + 1e-6) * D ** -0.5
    k = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
    beta = torch.sigmoid(h @ W["b"].T)
    decay = torch.exp(-torch.exp(W["A_log"]) * softplus(h @ W["a"].T + W["dt_bias"]))
    S = torch.zeros(H, D, Dv, dtype=F64)
    o = torch.zeros(n, H, Dv, dtype=F64)
    for t in range(n):
        for hd in range(H):
            g = hd // (H // G)
            S[hd] = decay[t, hd] * S[hd]
            u = beta[t, hd] * (v[t, hd] - k[t, g] @ S[hd])
            S[hd] = S[hd] + torch.outer(k[t, g], u)
            o[t, hd] = q[t, g] @ S[hd]
    o = unit_rms(o, eps) * W["norm"]
    return (o.reshape(n, H * Dv) * silu(h @ W["g"].T)) @ W["o"].T


def latent_attention(h, W, m, eps):
    """Queries through a latent of their own; keys and values of every head from one normed latent per token plus one
    rotated key part shared by the heads; a sliding window."""
    n, H, D, R, Dv, C = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = ((unit_rms(h @ W["dq"].T, eps) * W["dq.norm"]) @ W["uq"].T).view(n, H, D + R)
    kv = h @ W["dkv"].T
    c = unit_rms(kv[:, :C], eps) * W["dkv.norm"]
    k_rot = rotate(kv[:, None, C:], m.get("rot"), True)[:, 0]
    q_rot = rotate(q[:, :, D:], m.get("rot"), True)
    k = (c @ W["uk"].T).view(n, H, D)
    v = (c @ W["uv"].T).view(n, H, Dv)
    see = visible(n, in_window, m)
    out = torch.zeros(n, H, Dv, dtype=F64)
    for hd in range(H):
        s = (q[:, hd, :D] @ k[:, hd].T + q_rot[:, hd] @ k_rot.T) * m["scale"]
        out[:, hd] = torch.softmax(s.masked_fill(~see, -float("inf")), -1) @ v[:, hd]
    return out.reshape(n, H * Dv) @ W["o"].T


def chunk_attention(h, W, m, eps):
    """Grouped-query attention inside fixed blocks of positions; q, k and v carry biases and pass a short convolution
    each; q and k are normed over all their rows at once, then rotated."""
    n, H, G, D, Dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (causal_conv(h @ W[c].T + W[c + ".b"], W[c + ".conv"]) for c in ("q", "k", "v"))
    q = rotate((unit_rms(q, eps) * W["q.norm"]).view(n, H, D), m.get("rot"), False)
    k = rotate((unit_rms(k, eps) * W["k.norm"]).view(n, G, D), m.get("rot"), False)
    v = v.view(n, G, Dv)
    see = visible(n, in_chunk, m)
    out = torch.zeros(n, H, Dv, dtype=F64)
    for hd in range(H):
        g = hd // (H // G)
        s = (q[:, hd] @ k[:, g].T) * m["scale"]
        out[:, hd] = torch.softmax(s.masked_fill(~see, -float("inf")), -1) @ v[:, g]
    return out.reshape(n, H * Dv) @ W["o"].T


# --------------------------------------------------------------------------------------------- feed-forward
def dense(h, W, f):
    return (silu(h @ W["gate"].T) * (h @ W["up"].T)) @ W["down"].T


def expert(h, W):
    return gelu(h @ W["up"].T) @ W["down"].T


def route(z, top):
    """[(expert, weight)] of one token: softmax over all experts, the `top` largest, divided by their sum."""
    s = torch.exp(z - z.max())
    s = s / s.sum()
    order = sorted(range(len(s)), key=lambda e: (-float(s[e]), e))[:top]
    total = sum(float(s[e]) for e in order) + 1e-20
    return [(e, float(s[e]) / total) for e in order]


def moe(h, W, f):
    z = h @ W["router"].T
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in route(z[t], f["router"]["top"]):
            y[t] += w * expert(h[t], sub(W, f"e{e}."))
    return y + expert(h, sub(W, "shared.")) if f.get("shared") else y


# --------------------------------------------------------------------------------------------- model
MIXERS = {"delta": gated_delta, "latent_attention": latent_attention, "attention": chunk_attention}
FEED_FORWARDS = {"dense": dense, "moe": moe}


def sub(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def order(cfg):
    """Layer indices in the order they run: the looped span several times in a row."""
    L, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(L))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, L))


def forward(cfg, tensors, tokens):
    """Returns (logits [n, V], residual stream after every layer run [runs, n, E])."""
    T = {k: v.to(F64) for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    x = T["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"]
    after = []
    for i in order(cfg):
        ent, L = cfg["layers"][i], sub(T, f"l{i}.")
        x = x + MIXERS[ent["type"]](centred_norm(x, L["norm1"], eps), sub(L, "mix."), ent["mixer"], eps)
        f = ent.get("mlp")
        if f:
            x = x + FEED_FORWARDS[f["kind"]](centred_norm(x, L["norm2"], eps), sub(L, "mlp."), f)
        after.append(x.clone())
    return centred_norm(x, T["final.norm"], eps) @ T["head"].T, torch.stack(after)
