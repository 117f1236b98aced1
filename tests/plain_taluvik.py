"""A plain, slow implementation of the Taluvik decoder, one function per mechanism, in float64 on the CPU.

It shares no code with the product.  ``weights`` maps tensor names to tensors; ``config`` is the dictionary of
``config.json``.  A whole sequence is computed at once with explicit loops over tokens, heads and keys, so nothing
here knows of pages, slots, steps or batches.

Notation: ``h`` [T, width] is a mixer's or feed-forward's input, ``pos`` the tokens' positions 0..T-1.
"""
from __future__ import annotations

import math

import torch

F = torch.float64


# ---- small pieces -------------------------------------------------------------------------------
def layer_norm(x, w, b, eps):
    """The row's mean is taken off, the rest divided by sqrt(mean of its squares + eps), then weight and bias."""
    centred = x - x.mean(-1, keepdim=True)
    return centred / torch.sqrt((centred * centred).mean(-1, keepdim=True) + eps) * w + b


def rms_scale(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit_rows(x):
    """x / sqrt(sum of squares + 1e-6) over the last axis."""
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def silu(z):
    return z / (1.0 + torch.exp(-z))


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def causal_conv(x, taps, bias=None):
    """Per channel: out[t] = sum_j taps[:, j] x[t - (K - 1) + j] (+ bias), zeros ahead of the sequence."""
    T, C = x.shape
    K = taps.shape[1]
    out = torch.zeros(T, C, dtype=F)
    for t in range(T):
        for j in range(K):
            at = t - (K - 1) + j
            if at >= 0:
                out[t] += taps[:, j] * x[at]
    return out if bias is None else out + bias


def frequencies(dims: int, base: float, scaling: dict | None) -> list[float]:
    """f_i = base^(-2i / dims); with ``scaling`` {factor, low, high, original}: waves that turn more than ``high``
    times over ``original`` positions keep f, those that turn less than ``low`` times get f / factor, and between
    the two the share of f grows linearly with the number of turns."""
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling:
            length = 2.0 * math.pi / f
            turns = scaling["original"] / length
            if length > scaling["original"] / scaling["low"]:
                f = f / scaling["factor"]
            elif length >= scaling["original"] / scaling["high"]:
                s = (turns - scaling["low"]) / (scaling["high"] - scaling["low"])
                f = (1.0 - s) * f / scaling["factor"] + s * f
        out.append(f)
    return out


def turn_halves(x, pos, freqs):
    """x [T, heads, d]: dimension i turns with dimension i + n (n frequencies) by pos * f_i; the rest passes."""
    n = len(freqs)
    out = x.clone()
    for t, p in enumerate(pos):
        for i, f in enumerate(freqs):
            c, s = math.cos(p * f), math.sin(p * f)
            u, v = x[t, :, i], x[t, :, i + n]
            out[t, :, i] = u * c - v * s
            out[t, :, i + n] = v * c + u * s
    return out


def sees(p: int, j: int, size: int | None) -> bool:
    return j <= p and (not size or p // size == j // size)


def capped(score, cap):
    return cap * torch.tanh(score / cap) if cap else score


# ---- the mixers ----------------------------------------------------------------------------------
def attention(h, pos, W, pre, m, eps):
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = (h @ W[pre + "q"].T).view(T, H, d)
    k = (h @ W[pre + "k"].T).view(T, G, d)
    v = (h @ W[pre + "v"].T).view(T, G, dv)
    if m.get("rot"):
        freqs = frequencies(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling"))
        q, k = turn_halves(q, pos, freqs), turn_halves(k, pos, freqs)
    q, k = rms_scale(q, eps), rms_scale(k, eps)
    sink = W[pre + "sink"]
    size = (m.get("mask") or {}).get("size")
    out = torch.zeros(T, H, dv, dtype=F)
    for i in range(T):
        keys = [j for j in range(i + 1) if sees(pos[i], pos[j], size)]
        for a in range(H):
            g = a // (H // G)
            s = capped((k[keys, g] @ q[i, a]) * m["scale"], m.get("softcap"))
            top = max(float(s.max()), float(sink[a]))
            e = torch.exp(s - top)
            out[i, a] = (e @ v[keys, g]) / (e.sum() + math.exp(float(sink[a]) - top))
    return out.reshape(T, H * dv) @ W[pre + "o"].T


def delta(h, W, pre, m, eps):
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q, k, v = (silu(causal_conv(h @ W[pre + n].T, W[pre + n + ".conv"])) for n in "qkv")
    q = unit_rows(q.view(T, G, d)) * d ** -0.5
    k = unit_rows(k.view(T, G, d))
    v = v.view(T, H, dv)
    beta = torch.sigmoid(h @ W[pre + "b"].T)
    decay = torch.exp(-torch.exp(W[pre + "A_log"]) * softplus(h @ W[pre + "a"].T + W[pre + "dt_bias"]))
    out = torch.zeros(T, H, dv, dtype=F)
    for a in range(H):
        g = a // (H // G)
        S = torch.zeros(d, dv, dtype=F)
        for t in range(T):
            S = decay[t, a] * S
            u = beta[t, a] * (v[t, a] - S.T @ k[t, g])
            S = S + torch.outer(k[t, g], u)
            out[t, a] = S.T @ q[t, g]
    out = rms_scale(out, eps) * W[pre + "norm"] * silu(h @ W[pre + "g"].T).view(T, H, dv)
    return out.reshape(T, H * dv) @ W[pre + "o"].T


def mamba1(h, W, pre, m):
    inner, N, R = m["inner"], m["state"], m["dt_rank"]
    T = h.shape[0]
    xz = h @ W[pre + "in"].T
    x, z = xz[:, :inner], xz[:, inner:]
    x = silu(causal_conv(x, W[pre + "conv"], W[pre + "conv.b"]))
    low = x @ W[pre + "x"].T
    dt = softplus(low[:, :R] @ W[pre + "dt"].T + W[pre + "dt.b"])
    B, C = low[:, R:R + N], low[:, R + N:]
    A = -torch.exp(W[pre + "A_log"])
    S = torch.zeros(inner, N, dtype=F)
    y = torch.zeros(T, inner, dtype=F)
    for t in range(T):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + W[pre + "D"] * x[t]
    return (y * silu(z)) @ W[pre + "o"].T


def mixer(kind, h, pos, W, pre, m, eps):
    if kind == "attention":
        return attention(h, pos, W, pre, m, eps)
    if kind == "delta":
        return delta(h, W, pre, m, eps)
    if kind == "mamba1":
        return mamba1(h, W, pre, m)
    raise ValueError(kind)


def gated_ff(h, W, pre):
    return (gelu_tanh(h @ W[pre + "gate"].T) * (h @ W[pre + "up"].T)) @ W[pre + "down"].T


# ---- the model -----------------------------------------------------------------------------------
def as_double(weights):
    return {k: v.to(F) for k, v in weights.items()}


def owner(layers, i):
    """The layer whose tensors layer i runs on."""
    while layers[i].get("weights_of") is not None:
        i = layers[i]["weights_of"]
    return i


def forward(config, weights, tokens, stream=None):
    """Logits [T, vocab] of a whole sequence; ``stream`` (a list) gets the residual stream after every layer."""
    W = as_double(weights)
    eps, mult = config["norm"]["eps"], config["residual_mult"]
    pos = list(range(len(tokens)))
    x = W["embed"][torch.tensor(list(tokens))] * config["embedding"]["scale"]
    for i, layer in enumerate(config["layers"]):
        pre = f"l{owner(config['layers'], i)}."
        h = layer_norm(x, W[pre + "norm1"], W[pre + "norm1.b"], eps)
        y = mixer(layer["type"], h, pos, W, pre + "mix.", layer["mixer"], eps)
        if layer.get("mlp"):
            y = y + gated_ff(h, W, pre + "mlp.")
        x = x + mult * y
        if stream is not None:
            stream.append(x)
    return layer_norm(x, W["final.norm"], W["final.norm.b"], eps) @ W["head"].T
