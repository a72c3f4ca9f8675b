"""A plain, slow implementation of the Zotunex decoder: float64 on the CPU, whole sequences, no cache, one function
per mechanism.  It shares no code with the engine; the tests compare the engine against it.

Notation: h [T, width] is a sublayer's input for the T tokens of one sequence, positions 0 .. T-1; W are matrices
stored [out, in] and applied as h W^T; `t` is the dictionary of a model's tensors by name (float64).
"""

from __future__ import annotations

import math

import torch

F64 = torch.float64

_ROUND = None  # set while `forward(..., rounded=...)` runs


def operand(x):
    """An operand of a matrix product (a sublayer's input, what its last projection reads, queries, keys, values and
    latents): as it is, or rounded where `forward` was asked to show what rounding these operands alone does."""
    return x if _ROUND is None else _ROUND(x)


def rms(x, eps, weight=None):
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if weight is None else y * weight


# ------------------------------------------------------------------------------------------------ rotation
def frequencies(rot):
    """f_i = base^(-2i/dims), i < dims/2, all divided by scaling.factor where a scaling is given."""
    dims = int((rot or {}).get("dims", 0))
    f = torch.tensor([float(rot["base"]) ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F64)
    scaling = (rot or {}).get("scaling")
    return f / float(scaling["factor"]) if scaling else f


def rotate_neighbours(x, freq, positions):
    """x [T, heads, d]: dimensions 2i and 2i + 1 turn together by positions * freq[i]; the rest passes."""
    n = 2 * freq.numel()
    if n == 0:
        return x
    ang = positions.to(F64)[:, None] * freq[None, :]
    c, s = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    turned = torch.stack([u * c - v * s, v * c + u * s], dim=-1).flatten(-2)
    return torch.cat([turned, x[..., n:]], dim=-1)


def rotate_half(x, freq, positions):
    """x [T, heads, d]: dimension i < len(freq) turns together with dimension i + len(freq); the rest passes."""
    half = freq.numel()
    if half == 0:
        return x
    ang = positions.to(F64)[:, None] * freq[None, :]
    c, s = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], dim=-1)


# ------------------------------------------------------------------------------------------------ mixers
def causal(T):
    return torch.triu(torch.ones(T, T, dtype=torch.bool), 1)


def attention(h, t, p, m, eps):
    """Grouped softmax attention whose values are the projected keys: q and k are normed head by head with weights the
    heads share, then turned; the scores of a head carry a number of its own, and so does its result's gate.
    `m`: heads, kv_heads, dim, vdim (= dim), scale, rot {base, dims, scaling {factor}}."""
    T = h.shape[0]
    H, G, d = int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    q = (h @ t[p + "q"].T).view(T, H, d)
    k = (h @ t[p + "k"].T).view(T, G, d)
    v = operand(k)
    freq, pos = frequencies(m.get("rot")), torch.arange(T)
    q = operand(rotate_neighbours(rms(q, eps, t[p + "q.norm"]), freq, pos))
    k = operand(rotate_neighbours(rms(k, eps, t[p + "k.norm"]), freq, pos))
    gate = torch.sigmoid(h @ t[p + "g"].T)
    out = torch.zeros(T, H, d, dtype=F64)
    for a in range(H):
        g = a // (H // G)
        s = (q[:, a] @ k[:, g].T) * float(m["scale"]) * t[p + "temp"][a]
        w = torch.softmax(s.masked_fill(causal(T), -math.inf), dim=-1)
        out[:, a] = (w @ v[:, g]) * gate[:, a:a + 1]
    return operand(out.reshape(T, H * d)) @ t[p + "o"].T


def softmax_with_sink(s, sink):
    """Softmax over the last axis of s (masked keys are -inf) whose denominator also holds exp(sink)."""
    top = torch.clamp(s.max(-1, keepdim=True).values, min=float(sink))
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - top))


def latent_attention(h, t, p, m, eps):
    """Attention whose keys and values come from one latent per token and one turned key part for all heads, with a sink
    per head in the softmax and a gate per head on the result.  `m`: heads, dim, rot_dim, vdim, kv_rank, scale, rot."""
    T = h.shape[0]
    H, dn, dr, dv, r = int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"])
    freq, pos = frequencies(m.get("rot")), torch.arange(T)
    q = (h @ t[p + "q"].T).view(T, H, dn + dr)
    qn, qr = operand(q[..., :dn]), operand(rotate_half(q[..., dn:], freq, pos))
    kv = h @ t[p + "dkv"].T
    c = operand(rms(kv[:, :r], eps, t[p + "dkv.norm"]))
    kr = operand(rotate_half(kv[:, r:].reshape(T, 1, dr), freq, pos)[:, 0])
    kn = (c @ t[p + "uk"].T).view(T, H, dn)
    v = (c @ t[p + "uv"].T).view(T, H, dv)
    gate = torch.sigmoid(h @ t[p + "g"].T)
    out = torch.zeros(T, H, dv, dtype=F64)
    for a in range(H):
        s = (qn[:, a] @ kn[:, a].T + qr[:, a] @ kr.T) * float(m["scale"])
        w = softmax_with_sink(s.masked_fill(causal(T), -math.inf), t[p + "sink"][a])
        out[:, a] = (w @ v[:, a]) * gate[:, a:a + 1]
    return operand(out.reshape(T, H * dv)) @ t[p + "o"].T


# ------------------------------------------------------------------------------------------------ feed-forward
def squared_relu_unit(h, t, p):
    u = torch.clamp(h @ t[p + "up"].T, min=0.0)
    return operand(u * u) @ t[p + "down"].T


def clamped_unit(h, t, p, limit):
    g = torch.clamp(h @ t[p + "gate"].T, max=float(limit))
    u = torch.clamp(h @ t[p + "up"].T, min=-float(limit), max=float(limit))
    return operand(g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ t[p + "down"].T


def route(h, t, p, router):
    """(chosen experts [T, top], their weights): the largest of sigmoid scores plus a correction; the weights are the
    scores without it, times a constant."""
    s = torch.sigmoid(h @ t[p + "router"].T)
    idx = torch.topk(s + t[p + "correction"][None, :], int(router["top"]), dim=-1).indices
    return idx, torch.gather(s, 1, idx) * float(router["scale"])


def mixture(h, t, p, mlp):
    router, expert, shared = mlp["router"], mlp["expert"], mlp.get("shared")
    idx, w = route(h, t, p, router)
    y = torch.zeros(h.shape[0], t[p + "e0.down"].shape[0], dtype=F64)
    for e in range(int(router["experts"])):
        rows, col = torch.nonzero(idx == e, as_tuple=True)
        if rows.numel():
            y[rows] += w[rows, col][:, None] * clamped_unit(h[rows], t, f"{p}e{e}.", expert["limit"])
    if shared:
        y = y + clamped_unit(h, t, p + "shared.", shared["limit"])
    return y


# ------------------------------------------------------------------------------------------------ the model
def mixer(kind, h, t, p, m, eps):
    if kind == "attention":
        return attention(h, t, p, m, eps)
    if kind == "latent_attention":
        return latent_attention(h, t, p, m, eps)
    raise ValueError(kind)


def layer(x, t, i, entry, eps):
    p = f"l{i}."
    x = x + mixer(entry["type"], operand(rms(x, eps, t[p + "norm1"])), t, p + "mix.", entry["mixer"], eps)
    mlp = entry.get("mlp")
    if mlp is None:
        return x
    h = operand(rms(x, eps, t[p + "norm2"]))
    return x + (mixture(h, t, p + "mlp.", mlp) if mlp["kind"] == "moe" else squared_relu_unit(h, t, p + "mlp."))


def forward(config, t, tokens, collect=None, rounded=None):
    """Logits [T, vocab] of one sequence.  `collect`: a list that receives the residual stream after every layer.
    `rounded`: a function applied to the operands of matrix products (see `operand`)."""
    global _ROUND
    _ROUND = rounded
    try:
        eps = float(config["norm"]["eps"])
        x = t["embed"][torch.as_tensor(tokens, dtype=torch.long)] * float(config["embedding"]["scale"])
        for i, entry in enumerate(config["layers"]):
            x = layer(x, t, i, entry, eps)
            if collect is not None:
                collect.append(x.clone())
        return operand(rms(x, eps, t["final.norm"])) @ t["head"].T
    finally:
        _ROUND = None
