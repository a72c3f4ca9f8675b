"""A plain, slow implementation of the Ramolix decoder: float64 on the CPU, whole sequences, no cache, one function
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


def silu(x):
    return x * torch.sigmoid(x)


def softplus(x):
    return torch.where(x > 30, x, torch.log1p(torch.exp(torch.clamp(x, max=30))))


def gelu_tanh(x):
    return 0.5 * x * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (x + 0.044715 * x ** 3)))


# ------------------------------------------------------------------------------------------------ rotation
def frequencies(rot):
    """f_i = base^(-2i/dims), i < dims/2; with scaling {factor, low, high, original} long wavelengths are stretched:
    kept below original/high, divided by factor beyond original/low, blended in between."""
    rot = rot or {}
    dims, scaling, out = int(rot.get("dims", 0)), rot.get("scaling"), []
    for i in range(dims // 2):
        f = float(rot["base"]) ** (-2.0 * i / dims)
        if scaling:
            factor, low, high, orig = (float(scaling[k]) for k in ("factor", "low", "high", "original"))
            wave = 2.0 * math.pi / f
            if wave > orig / low:
                f = f / factor
            elif wave >= orig / high:
                s = (orig / wave - low) / (high - low)
                f = (1.0 - s) * f / factor + s * f
        out.append(f)
    return torch.tensor(out, dtype=F64)


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
def visible(T, window=None):
    """[T, T]: whether the query in a row sees the key in a column: itself and what came before it, the last `window`
    tokens of that where there is a window."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) if window is None else (j <= i) & (i - j < int(window))


def attention(h, t, p, m, eps):
    """Grouped softmax attention whose values are the projected keys: queries and keys are normed over all heads at once,
    then turned; a sliding window.  `m`: heads, kv_heads, dim, vdim (= dim), scale, mask {size}, rot {base, dims, scaling}."""
    T = h.shape[0]
    H, G, d = int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    q = h @ t[p + "q"].T + t[p + "q.b"]
    k = h @ t[p + "k"].T + t[p + "k.b"]
    v = operand(k.view(T, G, d))
    freq, pos = frequencies(m.get("rot")), torch.arange(T)
    q = operand(rotate_half(rms(q, eps, t[p + "q.norm"]).view(T, H, d), freq, pos))
    k = operand(rotate_half(rms(k, eps, t[p + "k.norm"]).view(T, G, d), freq, pos))
    seen = visible(T, (m.get("mask") or {}).get("size"))
    out = torch.zeros(T, H, d, dtype=F64)
    for a in range(H):
        g = a // (H // G)
        s = (q[:, a] @ k[:, g].T) * float(m["scale"])
        out[:, a] = torch.softmax(s.masked_fill(~seen, -math.inf), dim=-1) @ v[:, g]
    return operand(out.reshape(T, H * d)) @ t[p + "o"].T


def latents(h, t, p, eps):
    """The row a token keeps for all heads."""
    return operand(rms(h @ t[p + "dkv"].T, eps, t[p + "dkv.norm"]))


def latent_attention(h, c, t, p, m):
    """Causal attention whose keys and values are projections of the latents c [T, kv_rank] (this layer's own or an earlier
    layer's), without positions.  `m`: heads, dim, vdim, kv_rank, scale."""
    T = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = operand(h @ t[p + "q"].T).view(T, H, d)
    k = (c @ t[p + "uk"].T).view(T, H, d)
    v = (c @ t[p + "uv"].T).view(T, H, dv)
    out = torch.zeros(T, H, dv, dtype=F64)
    for a in range(H):
        s = (q[:, a] @ k[:, a].T) * float(m["scale"])
        out[:, a] = torch.softmax(s.masked_fill(~visible(T), -math.inf), dim=-1) @ v[:, a]
    return operand(out.reshape(T, H * dv)) @ t[p + "o"].T


def causal_conv(x, w, bias):
    """x [T, C], w [C, taps] with the last column for the present token; zeros before the sequence."""
    T, C = x.shape
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, C, dtype=x.dtype), x], dim=0)
    y = bias[None, :].expand(T, C).clone()
    for j in range(taps):
        y = y + padded[j:j + T] * w[:, j][None, :]
    return y


def state_space(x, B, C, dt, A, D):
    """The recurrence token by token.  x [T, H, P], B and C [T, G, N] (head h uses group h / (H / G)), dt [T, H], A and D [H]:
    S <- exp(A dt) S + dt B x^T;  y = S^T C + D x."""
    T, H, P = x.shape
    G, N = B.shape[1:]
    S = torch.zeros(H, N, P, dtype=F64)
    y = torch.zeros(T, H, P, dtype=F64)
    of = torch.arange(H) // (H // G)
    for i in range(T):
        b, c = B[i][of], C[i][of]
        S = torch.exp(A * dt[i])[:, None, None] * S + (dt[i][:, None] * b)[:, :, None] * x[i][:, None, :]
        y[i] = (S * c[:, :, None]).sum(1) + D[:, None] * x[i]
    return y


def gated_group_norm(y, z, weight, groups, eps):
    """y silu(z), each of `groups` equal parts of a row divided by its own root mean square, times a weight."""
    u = (y * silu(z)).view(y.shape[0], groups, -1)
    return rms(u, eps).reshape(y.shape) * weight[None, :]


def mamba2(h, t, p, m, eps):
    """A state-space mixer with one decay per head and token.  `m`: heads, vdim, state, groups, norm_groups."""
    T = h.shape[0]
    H, P, N, G = int(m["heads"]), int(m["vdim"]), int(m["state"]), int(m["groups"])
    inner = H * P
    zxbcdt = h @ t[p + "in"].T
    z, xbc, dt = zxbcdt[:, :inner], zxbcdt[:, inner:2 * inner + 2 * G * N], zxbcdt[:, 2 * inner + 2 * G * N:]
    xbc = operand(silu(causal_conv(xbc, t[p + "conv"], t[p + "conv.b"])))
    x, B, C = xbc[:, :inner].view(T, H, P), xbc[:, inner:inner + G * N].view(T, G, N), xbc[:, inner + G * N:].view(T, G, N)
    dt = softplus(dt + t[p + "dt_bias"][None, :])
    y = state_space(x, B, C, dt, -torch.exp(t[p + "A_log"]), t[p + "D"]).reshape(T, inner)
    return operand(gated_group_norm(y, z, t[p + "norm"], int(m["norm_groups"]), eps)) @ t[p + "o"].T


# ------------------------------------------------------------------------------------------------ feed-forward
def gelu_gated(h, t, p):
    return operand(gelu_tanh(h @ t[p + "gate"].T) * (h @ t[p + "up"].T)) @ t[p + "down"].T


# ------------------------------------------------------------------------------------------------ the model
def joined(x, y, weight, eps, mult):
    """The residual sum: a sublayer's result joins the stream through its norm."""
    return x + mult * rms(y, eps, weight)


def layer(x, t, i, entry, eps, mult, kept):
    """`kept`: the latents of the layers so far, by layer."""
    p, m, h = f"l{i}.", entry["mixer"], operand(x)
    if entry["type"] == "attention":
        y = attention(h, t, p + "mix.", m, eps)
    elif entry["type"] == "mamba2":
        y = mamba2(h, t, p + "mix.", m, eps)
    elif entry["type"] == "latent_attention":
        source = m.get("kv_from")
        if source is None:
            source = i
            kept[i] = latents(h, t, p + "mix.", eps)
        y = latent_attention(h, kept[source], t, p + "mix.", m)
    else:
        raise ValueError(entry["type"])
    x = joined(x, y, t[p + "norm1"], eps, mult)
    if entry.get("mlp") is None:
        return x
    return joined(x, gelu_gated(operand(x), t, p + "mlp."), t[p + "norm2"], eps, mult)


def forward(config, t, tokens, collect=None, rounded=None):
    """Logits [T, vocab] of one sequence.  `collect`: a list that receives the residual stream after every layer.
    `rounded`: a function applied to the operands of matrix products (see `operand`)."""
    global _ROUND
    _ROUND = rounded
    try:
        eps, mult = float(config["norm"]["eps"]), float(config["residual_mult"])
        x = t["embed"][torch.as_tensor(tokens, dtype=torch.long)] * float(config["embedding"]["scale"])
        kept = {}
        for i, entry in enumerate(config["layers"]):
            x = layer(x, t, i, entry, eps, mult, kept)
            if collect is not None:
                collect.append(x.clone())
        return operand(rms(x, eps, t["final.norm"])) @ t["embed"].T
    finally:
        _ROUND = None
