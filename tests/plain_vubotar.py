"""A plain, slow implementation of the Vubotar decoder, one function per mechanism, in float64 on the CPU.

It shares no code with the product.  ``weights`` maps tensor names to tensors; ``config`` is the dictionary of
``config.json``.  A whole sequence is computed at once, so nothing here knows of pages, slots, steps or batches.

Notation: ``h`` [T, width] is a mixer's or feed-forward's input, ``pos`` the tokens' positions 0..T-1, ``W`` the weights
in double precision, ``p`` the prefix of a part's tensor names.
"""
from __future__ import annotations

import math

import torch

F = torch.float64


# ---- small pieces -------------------------------------------------------------------------------
def rms_scale(x, eps):
    """Every row of the last axis over the root of its mean square, ``eps`` added inside the root."""
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return rms_scale(x, eps) * w


def silu(z):
    return z / (1.0 + torch.exp(-z))


def log_sigmoid(z: float) -> float:
    return -math.log1p(math.exp(-z)) if z > 0 else z - math.log1p(math.exp(z))


def bend(s, cap):
    """``cap * tanh(s / cap)``; no cap: s."""
    return cap * torch.tanh(s / cap) if cap else s


def turn_pairs(x, pos, dims: int, base: float):
    """x [T, ..., n]: entries 2i and 2i + 1 of the first ``dims`` turn by ``pos * base^(-2i / dims)``; the rest passes."""
    out = x.clone()
    for t, at in enumerate(pos):
        for i in range(dims // 2):
            a = at * base ** (-2.0 * i / dims)
            c, s = math.cos(a), math.sin(a)
            u, v = x[t, ..., 2 * i], x[t, ..., 2 * i + 1]
            out[t, ..., 2 * i] = u * c - v * s
            out[t, ..., 2 * i + 1] = v * c + u * s
    return out


def bucket(n: int, rows: int, reach: int) -> int:
    """The row of a distance table of ``rows`` rows for distance n: the first half of the rows one per distance, the
    others on a logarithmic scale up to ``reach``.  In whole numbers: the log-scaled row is the largest k with
    (reach / half)^k <= (n / half)^(rows - half)."""
    half = rows // 2
    if n < half:
        return n
    rest = rows - half
    k = 0
    while half + k < rows - 1 and reach ** (k + 1) * half ** rest <= n ** rest * half ** (k + 1):
        k += 1
    return half + k


def sees(i: int, j: int, mask: dict | None) -> bool:
    """Whether the token at i sees the key at j: not ahead, and either in the window or among the kept first."""
    if j > i:
        return False
    return mask is None or i - j < mask["size"] or j < mask.get("keep_first", 0)


# ---- the mixers ----------------------------------------------------------------------------------
def attention_weights(s, visible, one_more: bool):
    """Softmax of the visible scores of each row; with ``one_more`` a 1 joins the denominator."""
    s = s.masked_fill(~visible, -math.inf)
    top = s.max(1, keepdim=True).values
    if one_more:
        top = top.clamp(min=0.0)
    e = torch.exp(s - top)
    total = e.sum(1, keepdim=True)
    return e / (total + torch.exp(-top) if one_more else total)


def mixer_latent(h, pos, W, p: str, m: dict, eps: float):
    """Queries through a normed latent; keys and values of all heads out of another normed latent; one turned key part
    for all heads; a gate per output column."""
    T, H, d, dr, dv, r = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    base = m["rot"]["base"]
    q = (rms_norm(h @ W[p + "dq"].T, W[p + "dq.norm"], eps) @ W[p + "uq"].T).view(T, H, d + dr)
    down = h @ W[p + "dkv"].T
    c = rms_norm(down[:, :r], W[p + "dkv.norm"], eps)
    key_turned = turn_pairs(down[:, r:], pos, dr, base)
    q_turned = turn_pairs(q[:, :, d:], pos, dr, base)
    key_plain, value = (c @ W[p + "uk"].T).view(T, H, d), (c @ W[p + "uv"].T).view(T, H, dv)
    visible = torch.tensor([[j <= i for j in pos] for i in pos])
    heads = []
    for a in range(H):
        s = (q[:, a, :d] @ key_plain[:, a].T + q_turned[:, a] @ key_turned.T) * m["scale"]
        heads.append(attention_weights(s, visible, one_more=False) @ value[:, a])
    return (torch.cat(heads, 1) * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def attention_values(h, W, p: str, m: dict, first):
    """A layer's values [T, kv_heads * vdim], mixed with the first mixing layer's where the layer mixes; ``first`` is
    None (this is that first layer, or the layer does not mix) or those values."""
    v = h @ W[p + "v"].T
    if m.get("v_mix") and first is not None:
        lam = float(W[p + "vmix"])
        v = (1.0 - lam) * v + lam * first
    return v


def mixer_attention(h, pos, W, p: str, m: dict, eps: float, first=None):
    """Grouped heads without rotation: normed q and k per head, capped scores plus a bias by distance, a window that
    keeps the first tokens, a one in the denominator."""
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm((h @ W[p + "q"].T).view(T, H, d), W[p + "q.norm"], eps)
    k = rms_norm((h @ W[p + "k"].T).view(T, G, d), W[p + "k.norm"], eps)
    v = attention_values(h, W, p, m, first).view(T, G, dv)
    mask = m.get("mask")
    visible = torch.tensor([[sees(i, j, mask) for j in pos] for i in pos])
    table = W[p + "rel"]
    rows = [bucket(n, table.shape[0], m["bias_max"]) for n in range(T)]
    at = torch.tensor([[rows[max(i - j, 0)] for j in pos] for i in pos])
    heads = []
    for a in range(H):
        g = a // (H // G)
        s = bend((q[:, a] @ k[:, g].T) * m["scale"], m.get("softcap")) + table[at, a]
        heads.append(attention_weights(s, visible, one_more=True) @ v[:, g])
    return torch.cat(heads, 1) @ W[p + "o"].T


def mlstm_walk(q, k, v, i_log, f_log):
    """One head's matrix memory, token by token: q, k [T, d], v [T, dv], the two log gates [T].  Returns o [T, dv]."""
    T, d, dv = q.shape[0], q.shape[1], v.shape[1]
    S, n, m = torch.zeros(d, dv, dtype=F), torch.zeros(d, dtype=F), 0.0
    out = torch.zeros(T, dv, dtype=F)
    for t in range(T):
        i, f = float(i_log[t]), float(f_log[t])
        new = max(f + m, i)
        keep, add = math.exp(f + m - new), math.exp(i - new)
        m = new
        S = keep * S + add * torch.outer(k[t], v[t])
        n = keep * n + add * k[t]
        out[t] = (q[t] @ S) / (max(abs(float(n @ q[t])), math.exp(-m)) + 1e-6)
    return out


def mlstm_gates(h, W, p: str, cap: float):
    """(log input gates, log forget gates), each [T, heads]."""
    i = bend(h @ W[p + "i"].T + W[p + "i.b"], cap)
    f = bend(h @ W[p + "f"].T + W[p + "f.b"], cap)
    return i, torch.tensor([[log_sigmoid(float(z)) for z in row] for row in f], dtype=F)


def mixer_mlstm(h, W, p: str, m: dict, eps: float):
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ W[p + "q"].T).view(T, H, d) * d ** -0.5
    k = (h @ W[p + "k"].T).view(T, H, d)
    v = (h @ W[p + "v"].T).view(T, H, dv)
    i, f = mlstm_gates(h, W, p, m["gate_cap"])
    o = torch.stack([mlstm_walk(q[:, a], k[:, a], v[:, a], i[:, a], f[:, a]) for a in range(H)], 1)
    o = rms_scale(o, eps).reshape(T, H * dv) * W[p + "norm"]
    return (o * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


# ---- feed-forward ---------------------------------------------------------------------------------
def gated_ff(h, W, p: str):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def route(z, correction, top: int) -> tuple[list[int], list[float]]:
    """One token's router logits -> (chosen experts, their weights): chosen by sigmoid(z) + correction, weighted by
    sigmoid(z) alone over the chosen ones' sum."""
    s = torch.sigmoid(z)
    by = [float(a) for a in s + correction]
    chosen = sorted(range(len(by)), key=lambda e: (-by[e], e))[:top]
    return chosen, shares(s, chosen)


def shares(s, chosen) -> list[float]:
    total = sum(float(s[e]) for e in chosen) + 1e-20
    return [float(s[e]) / total for e in chosen]


def ff_experts(h, W, p: str, mlp: dict, forced=None, seen=None):
    """``forced``: per token the experts to use instead of the router's own choice (their weights still come from the
    scores).  ``seen``: a list that gets the router's logits [T, experts]."""
    out = torch.zeros_like(h)
    z = h @ W[p + "router"].T
    if seen is not None:
        seen.append(z.clone())
    for t in range(h.shape[0]):
        if forced is not None:
            chosen = [int(e) for e in forced[t]]
            weights = shares(torch.sigmoid(z[t]), chosen)
        else:
            chosen, weights = route(z[t], W[p + "correction"], mlp["router"]["top"])
        for e, w in zip(chosen, weights):
            out[t] += w * gated_ff(h[t:t + 1], W, f"{p}e{e}.")[0]
    return out


def is_close_call(z, correction, taken, mlp: dict, slack: float) -> bool:
    """Whether the experts ``taken`` are what the router chooses once every logit may move by up to ``slack``: tried with
    theirs up and the others down."""
    move = torch.full((z.shape[0],), -slack, dtype=F)
    for e in taken:
        move[int(e)] = slack
    return sorted(route(z + move, correction, mlp["router"]["top"])[0]) == sorted(int(e) for e in taken)


# ---- the model ------------------------------------------------------------------------------------
def as_double(weights: dict) -> dict:
    return {k: v.to(F) for k, v in weights.items() if v.dtype.is_floating_point}


def mixer(kind: str, h, pos, W, p: str, m: dict, eps: float, first=None):
    if kind == "attention":
        return mixer_attention(h, pos, W, p, m, eps, first)
    if kind == "latent_attention":
        return mixer_latent(h, pos, W, p, m, eps)
    if kind == "mlstm":
        return mixer_mlstm(h, W, p, m, eps)
    raise ValueError(kind)


def head(x, W, config: dict):
    z = (rms_norm(x, W["final.norm"], config["norm"]["eps"]) @ W["head"].T) * config.get("logit_scale", 1.0)
    return bend(z, config.get("logit_softcap"))


def forward(config: dict, weights: dict, tokens, forced_experts=None, want_layers: bool = False, router_logits=None):
    """Logits [T, vocab] of one sequence from position 0 (and the stream after every layer, if asked).
    ``forced_experts``: {layer index: per token the experts to use}; ``router_logits``: a dictionary that gets
    {layer index: the router's logits [T, experts]}."""
    W = as_double(weights)
    eps = config["norm"]["eps"]
    pos = list(range(len(tokens)))
    x = W["embed"][torch.tensor(tokens, dtype=torch.long)] * config.get("embedding", {}).get("scale", 1.0)
    after, first = [], None
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = rms_norm(x, W[p + "norm1"], eps)
        y = mixer(layer["type"], h, pos, W, p + "mix.", m, eps, first) * W[p + "ls1"]
        if layer["type"] == "attention" and m.get("v_mix") and first is None:
            first = attention_values(h, W, p + "mix.", m, None)
        mlp = layer.get("mlp")
        if mlp is not None:
            seen = [] if router_logits is not None else None
            g = rms_norm(x, W[p + "norm2"], eps)
            y = y + ff_experts(g, W, p + "mlp.", mlp, None if forced_experts is None else forced_experts.get(i), seen) * W[p + "ls2"]
            if seen:
                router_logits[i] = seen[0]
        x = x + y
        after.append(x.clone())
    logits = head(x, W, config)
    return (logits, torch.stack(after)) if want_layers else logits
