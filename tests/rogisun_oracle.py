"""Plain, slow float64 implementation of the Rogisun design, one function per mechanism.

It is the yardstick of the Rogisun tests and shares no code with the engine: it takes a config dict (the
layout of config.json) and a dict name -> torch tensor, runs one whole sequence at a time and keeps no cache
(attention looks at the whole prefix, recurrences are walked token by token from a zero state, convolutions
see zeros before the first token).

Notation: n tokens, width E. Linear weights are [out, in]; y = x @ W.T. A layer is
x <- x + mixer(conv1(N1(x))), then x <- x + ff(conv2(N2(x))), where N is an RMS norm with a weight vector and
conv(h) = h + causal_conv(h).
"""
from __future__ import annotations

import torch

F64 = torch.float64


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return unit_rms(x, eps) * w


def silu(z):
    return z * torch.sigmoid(z)


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


def input_conv(h, w):
    return h + causal_conv(h, w)


# --------------------------------------------------------------------------------------------- mixers
def lightning(h, W, m, eps):
    """Linear attention with one constant decay per head; silu on queries, keys and values; ONE RMS norm over the
    concatenated heads; a sigmoid gate."""
    n, H, D, Dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = silu(h @ W["q"].T).view(n, H, D)
    k = silu(h @ W["k"].T).view(n, H, D)
    v = silu(h @ W["v"].T).view(n, H, Dv)
    decay = torch.tensor(m["decay"], dtype=F64)
    S = torch.zeros(H, D, Dv, dtype=F64)
    o = torch.zeros(n, H, Dv, dtype=F64)
    for t in range(n):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    o = rms_norm(o.reshape(n, H * Dv), W["norm"], eps)
    return (o * torch.sigmoid(h @ W["g"].T)) @ W["o"].T


def mamba2(h, W, m, eps):
    """State-space layer: a scalar decay exp(-exp(A_log) dt) per head, inputs scaled by dt = softplus(.); x, B and C
    behind one short convolution with bias and silu; gate before the grouped norm."""
    n, H, Dv, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * Dv
    z, xbc, dt = torch.split(h @ W["in"].T, [inner, inner + 2 * G * N, H], dim=1)
    xbc = silu(causal_conv(xbc, W["conv"]) + W["conv.b"])
    x = xbc[:, :inner].reshape(n, H, Dv)
    Bm = xbc[:, inner:inner + G * N].reshape(n, G, N)
    Cm = xbc[:, inner + G * N:].reshape(n, G, N)
    dt = softplus(dt + W["dt_bias"])
    S = torch.zeros(H, N, Dv, dtype=F64)
    y = torch.zeros(n, H, Dv, dtype=F64)
    for t in range(n):
        for hd in range(H):
            g = hd // (H // G)
            a = torch.exp(-torch.exp(W["A_log"][hd]) * dt[t, hd])
            S[hd] = a * S[hd] + dt[t, hd] * torch.outer(Bm[t, g], x[t, hd])
            y[t, hd] = Cm[t, g] @ S[hd] + W["D"][hd] * x[t, hd]
    y = y.reshape(n, inner) * silu(z)
    parts = m["norm_groups"]
    y = unit_rms(y.reshape(n, parts, inner // parts), eps).reshape(n, inner) * W["norm"]
    return y @ W["o"].T


def visible(n, size):
    """Position i sees j <= i of the same block of `size` positions, blocks counted from position 0."""
    i = torch.arange(n)
    return (i[None, :] <= i[:, None]) & (i[None, :] // size == i[:, None] // size)


def chunk_attention(h, W, m, eps):
    """Grouped-query softmax attention inside fixed chunks of positions: values divided by their root mean square, a
    linear distance penalty per head, one sigmoid gate per head."""
    n, H, G, D, Dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ W["q"].T).view(n, H, D)
    k = (h @ W["k"].T).view(n, G, D)
    v = unit_rms((h @ W["v"].T).view(n, G, Dv), eps)
    gate = torch.sigmoid(h @ W["g"].T)
    i = torch.arange(n, dtype=F64)
    dist = i[:, None] - i[None, :]
    see = visible(n, m["mask"]["size"])
    out = torch.zeros(n, H, Dv, dtype=F64)
    for hd in range(H):
        g = hd // (H // G)
        s = (q[:, hd] @ k[:, g].T) * m["scale"] - 2.0 ** (-8.0 * (hd + 1) / H) * dist
        p = torch.softmax(s.masked_fill(~see, -float("inf")), -1)
        out[:, hd] = (p @ v[:, g]) * gate[:, hd:hd + 1]
    return out.reshape(n, H * Dv) @ W["o"].T


def gated_delta(h, W, m, eps):
    """Delta rule with a decay per head and key channel: the state forgets, then what it would answer to the new key is
    taken off the new value (times beta) before it is written, then it is read."""
    n, H, G, D, Dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = silu(causal_conv(h @ W["q"].T, W["q.conv"])).view(n, G, D)
    k = silu(causal_conv(h @ W["k"].T, W["k.conv"])).view(n, G, D)
    v = silu(causal_conv(h @ W["v"].T, W["v.conv"])).view(n, H, Dv)
    q = q / torch.sqrt((q * q).sum(-1, keepdim=True) + 1e-6) * D ** -0.5
    k = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
    beta = torch.sigmoid(h @ W["b"].T)
    low = softplus((h @ W["a1"].T) @ W["a2"].T + W["dt_bias"]).view(n, H, D)
    decay = torch.exp(-torch.exp(W["A_log"])[None, :, None] * low)
    S = torch.zeros(H, D, Dv, dtype=F64)
    o = torch.zeros(n, H, Dv, dtype=F64)
    for t in range(n):
        for hd in range(H):
            g = hd // (H // G)
            S[hd] = decay[t, hd][:, None] * S[hd]
            u = beta[t, hd] * (v[t, hd] - k[t, g] @ S[hd])
            S[hd] = S[hd] + torch.outer(k[t, g], u)
            o[t, hd] = q[t, g] @ S[hd]
    o = unit_rms(o, eps) * W["norm"]
    gate = torch.sigmoid((h @ W["g1"].T) @ W["g2"].T)
    return (o.reshape(n, H * Dv) * gate) @ W["o"].T


def parallel(h, W, m, eps):
    return (m["left_scale"] * chunk_attention(h, sub(W, "left."), m["left"], eps)
            + m["right_scale"] * gated_delta(h, sub(W, "right."), m["right"], eps))


# --------------------------------------------------------------------------------------------- feed-forward
def expert(h, W, limit):
    g = torch.clamp(h @ W["gate"].T, max=limit)
    u = torch.clamp(h @ W["up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ W["down"].T


def route(z, top):
    """[(expert, weight)] of one token: the `top` largest sigmoid scores, as they are."""
    s = torch.sigmoid(z)
    order = sorted(range(len(s)), key=lambda e: (-float(s[e]), e))[:top]
    return [(e, float(s[e])) for e in order]


def moe(h, W, f):
    z = h @ W["router"].T
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in route(z[t], f["router"]["top"]):
            y[t] += expert(w * h[t], sub(W, f"e{e}."), f["expert"]["limit"])
    return y


# --------------------------------------------------------------------------------------------- model
MIXERS = {"lightning": lightning, "mamba2": mamba2, "parallel": parallel}


def sub(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def forward(cfg, tensors, tokens):
    """Returns (logits [n, V], residual stream after every layer [L, n, E])."""
    T = {k: v.to(F64) for k, v in tensors.items()}
    eps = cfg["norm"]["eps"]
    x = T["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    after = []
    for i, ent in enumerate(cfg["layers"]):
        L = sub(T, f"l{i}.")
        x = x + MIXERS[ent["type"]](input_conv(rms_norm(x, L["norm1"], eps), L["canon1"]), sub(L, "mix."), ent["mixer"], eps)
        if ent.get("mlp"):
            x = x + moe(input_conv(rms_norm(x, L["norm2"], eps), L["canon2"]), sub(L, "mlp."), ent["mlp"])
        after.append(x.clone())
    return rms_norm(x, T["final.norm"], eps) @ T["embed"].T, torch.stack(after)
