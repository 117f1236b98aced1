"""Mixers that keep a matrix state per head and request instead of a cache of tokens.

The first ones run on one kernel (``kernels.linear_recurrence``): the state S [heads, key dim, value dim]
lives in float32 in the request's state slot, starts at zero, and is carried from token to token
and from step to step; a prompt portion is walked token by token in the order of the sequence.
``ssd``, ``gated_delta``, ``selective_scan`` and ``matrix_lstm`` take prompt portions in chunks of tokens instead.

``lightning_attention``: linear attention with a fixed decay per head.  With q = silu(W_q h), k =
silu(W_k h), v = silu(W_v h):  S_t = decay_h S_(t-1) + k_t v_t^T,  o_t = S_t^T q_t;  the heads'
outputs side by side are RMS-normed as one vector, multiplied by sigmoid(W_g h) and projected.

``wkv``: time mixing in the manner of RWKV (Peng et al., "RWKV: Reinventing RNNs for the Transformer
Era", and its later versions with a data-dependent decay).  Each of r, k, v, g, w reads its own mix of
the token's input and the previous token's, h + (h' - h) mu_s.  The decay is per token and key
channel, w_t = exp(-exp(W_w2 tanh(W_w1 mix_w) + w0));  o_t = (S_(t-1) + diag(u) k_t v_t^T)^T r_t,  S_t =
diag(w_t) S_(t-1) + k_t v_t^T.  Each head's output is divided by its own root mean square, then times
a weight and the gate silu(W_g mix_g), then projected.  The previous token's input is part of the
state: it sits behind S in the request's slot.
"""
from __future__ import annotations

import math

import torch

from tensorline_amd.ops import kernels
from tensorline_amd.parts.base import Linear, Part, TensorGetter, fuse_linears
from tensorline_amd.parts.registry import register_mixer
from tensorline_amd.parts.spec import StateNeed, TensorDecl


def _check_key_dim(prefix: str, dk: int) -> None:
    if dk <= 0 or dk > 256:
        raise ValueError(f"{prefix}: a key size of {dk} per head is not served: the recurrence kernel takes up to 256")


@register_mixer("lightning_attention")
class LightningAttention(Part):
    """Parameters: ``heads``, ``dim`` (query/key size per head), ``vdim``, ``decay`` (one per head),
    ``eps``.  Tensors under the prefix: q, k, v, g, o, norm."""

    def __init__(self, hidden_size, prefix, dtype, device, heads: int, dim: int, vdim: int, decay, eps: float):
        super().__init__(hidden_size, prefix, dtype, device)
        self.heads, self.dim, self.vdim, self.eps = int(heads), int(dim), int(vdim), float(eps)
        _check_key_dim(prefix, self.dim)
        if len(decay) != self.heads:
            raise ValueError(f"{prefix}: {len(decay)} decays for {self.heads} heads")
        self.decay = torch.tensor([float(d) for d in decay], dtype=torch.float32, device=device)
        H = self.heads
        mk = lambda s, n_out: Linear(prefix + s, hidden_size, n_out, False, weight_name=prefix + s)
        self._parts = [mk("q", H * self.dim), mk("k", H * self.dim), mk("v", H * self.vdim), mk("g", H * self.vdim)]
        self.proj: Linear | None = None
        self.o_proj = Linear(prefix + "o", H * self.vdim, hidden_size, False, weight_name=prefix + "o")
        self.norm_w = None

    def tensors(self):
        out = {}
        for p in self._parts + [self.o_proj]:
            out.update(p.tensors())
        out[self.prefix + "norm"] = TensorDecl((self.heads * self.vdim,), "one_plus_normal", 0.1, "float32")
        return out

    def load(self, get: TensorGetter) -> None:
        for p in self._parts + [self.o_proj]:
            p.load(get)
        self.proj = fuse_linears(self.prefix + "qkvg", self._parts)
        for p in self._parts:
            p.weight = None
        self.o_proj.prepare()
        self.norm_w = get(self.prefix + "norm")

    def weight_tensors(self):
        return self.proj.tensors_kept() + self.o_proj.tensors_kept() + [self.norm_w]

    def library_products(self):
        return [(self.proj.weight, torch.float32), (self.o_proj.weight, torch.float32)]

    def cache_need(self):
        return None

    def state_need(self):
        return StateNeed((self.heads * self.dim * self.vdim,), "float32")

    def forward(self, h, ctx, cache):
        H, dk, dv = self.heads, self.dim, self.vdim
        proj = self.proj(h, out_dtype=torch.float32)
        q, k = proj[:, :H * dk], proj[:, H * dk:2 * H * dk]
        v, g = proj[:, 2 * H * dk:2 * H * dk + H * dv], proj[:, 2 * H * dk + H * dv:]
        o = kernels.linear_recurrence(q, k, v, ctx, cache.state, H, dk, dv, decay=self.decay, silu_inputs=True)
        y = kernels.gated_group_norm(o, self.norm_w, g, H * dv, self.eps, "sigmoid", self.dtype)
        return self.o_proj(y, out_dtype=torch.float32)


@register_mixer("wkv")
class WKV(Part):
    """Parameters: ``heads``, ``dim`` (key and value size per head), ``eps``.  Tensors under the prefix:
    mu.r, mu.k, mu.v, mu.g, mu.w, r, k, v, g, w1, w2, w0, u, norm, o; the width of w1 / w2 (the
    decay's low-rank bottleneck) is read from ``decay_rank``."""

    WAYS = ("r", "k", "v", "g", "w")

    def __init__(self, hidden_size, prefix, dtype, device, heads: int, dim: int, decay_rank: int, eps: float):
        super().__init__(hidden_size, prefix, dtype, device)
        self.heads, self.dim, self.decay_rank, self.eps = int(heads), int(dim), int(decay_rank), float(eps)
        _check_key_dim(prefix, self.dim)
        N = self.heads * self.dim
        mk = lambda s, n_in, n_out, **kw: Linear(prefix + s, n_in, n_out, False, weight_name=prefix + s, **kw)
        self.r, self.k, self.v, self.g = (mk(s, hidden_size, N) for s in "rkvg")
        self.w1 = mk("w1", hidden_size, self.decay_rank)
        self.w2 = Linear(prefix + "w2", self.decay_rank, N, True, weight_name=prefix + "w2", bias_name=prefix + "w0")
        self.o_proj = mk("o", N, hidden_size)
        self.mu = self.u = self.norm_w = None

    def _linears(self):
        return [self.r, self.k, self.v, self.g, self.w1, self.w2, self.o_proj]

    def tensors(self):
        out = {}
        for p in self._linears():
            out.update(p.tensors())
        for s in self.WAYS:
            out[self.prefix + "mu." + s] = TensorDecl((self.hidden_size,), "normal", 0.3, "float32")
        out[self.prefix + "u"] = TensorDecl((self.heads, self.dim), "normal", 0.3, "float32")
        out[self.prefix + "norm"] = TensorDecl((self.heads * self.dim,), "one_plus_normal", 0.1, "float32")
        return out

    def load(self, get: TensorGetter) -> None:
        for p in self._linears():
            p.load(get)
            p.prepare()
        self.mu = torch.stack([get(self.prefix + "mu." + s) for s in self.WAYS]).contiguous()
        self.u = get(self.prefix + "u")
        self.norm_w = get(self.prefix + "norm")

    def weight_tensors(self):
        out = [self.mu, self.u, self.norm_w]
        for p in self._linears():
            out += p.tensors_kept()
        return out

    def library_products(self):
        return [(p.weight, torch.float32) for p in (self.r, self.g, self.o_proj)]

    def cache_need(self):
        return None

    def state_need(self):
        # the matrix state of every head, then the previous token's input
        return StateNeed((self.heads * self.dim * self.dim + self.hidden_size,), "float32")

    def forward(self, h, ctx, cache):
        H, d = self.heads, self.dim
        f32 = torch.float32
        mix = kernels.token_shift(h, self.mu, ctx, cache.state, H * d * d)          # [5, T, width]: r, k, v, g, w
        r, k, v, g = (lin(mix[i], out_dtype=f32) for i, lin in enumerate((self.r, self.k, self.v, self.g)))
        wlog = self.w2(kernels.tanh_rows(self.w1(mix[4], out_dtype=f32), self.dtype), out_dtype=f32)
        o = kernels.linear_recurrence(r, k, v, ctx, cache.state, H, d, d, wlog=wlog, bonus=self.u)
        y = kernels.gated_group_norm(o, self.norm_w, g, d, self.eps, "silu", self.dtype)
        return self.o_proj(y, out_dtype=f32)


@register_mixer("ssd")
class StateSpaceDuality(Part):
    """The mixer of Mamba-2 (Dao and Gu, "Transformers are SSMs: Generalized Models and Efficient
    Algorithms Through Structured State Space Duality").  Parameters: ``heads``, ``vdim`` (a head's
    channels), ``state`` (N), ``groups`` (heads of a group share B and C), ``conv`` (taps),
    ``norm_groups``, ``eps``.  With inner = heads * vdim, the input projection gives
    [z: inner | x: inner | B: groups*N | C: groups*N | dt: heads];  x, B and C pass a causal
    convolution per channel and SiLU;  dt = softplus(dt + dt_bias);  per head
    S_t = exp(-exp(A_log) dt) S_(t-1) + dt B_t x_t^T,  y_t = S_t^T C_t + D x_t;  y * silu(z) is RMS-normed in
    ``norm_groups`` equal parts, times ``norm``, and projected.  The request's slot keeps S [heads, N,
    vdim] and, behind it, the convolution's last ``conv`` - 1 inputs.  Tensors under the prefix: in,
    conv, conv.b, dt_bias, A_log, D, norm, o."""

    def __init__(self, hidden_size, prefix, dtype, device, heads: int, vdim: int, state: int, groups: int, conv: int,
                 norm_groups: int = 1, eps: float = 1e-6):
        super().__init__(hidden_size, prefix, dtype, device)
        self.heads, self.vdim, self.N, self.groups = int(heads), int(vdim), int(state), int(groups)
        self.taps, self.norm_groups, self.eps = int(conv), int(norm_groups), float(eps)
        _check_key_dim(prefix, self.N)
        self.inner = self.heads * self.vdim
        if self.groups <= 0 or self.heads % self.groups:
            raise ValueError(f"{prefix}: {heads} heads do not split into {groups} groups")
        if self.norm_groups <= 0 or self.inner % self.norm_groups:
            raise ValueError(f"{prefix}: {self.inner} channels do not split into {norm_groups} parts for the norm")
        if not 1 <= self.taps <= kernels.CONV_MAX_TAPS:
            raise ValueError(f"{prefix}: a convolution of {conv} taps is not served (1 to {kernels.CONV_MAX_TAPS})")
        self.conv_channels = self.inner + 2 * self.groups * self.N
        self.proj = Linear(prefix + "in", hidden_size, 2 * self.inner + 2 * self.groups * self.N + self.heads, False,
                           weight_name=prefix + "in")
        self.o_proj = Linear(prefix + "o", self.inner, hidden_size, False, weight_name=prefix + "o")
        self.conv_w = self.conv_b = self.dt_bias = self.rate_log = self.skip = self.norm_w = None

    def tensors(self):
        out = {**self.proj.tensors(), **self.o_proj.tensors()}
        p = self.prefix
        out[p + "conv"] = TensorDecl((self.conv_channels, self.taps), "normal", 0.3, "float32")
        out[p + "conv.b"] = TensorDecl((self.conv_channels,), "normal", 0.1, "float32")
        out[p + "dt_bias"] = TensorDecl((self.heads,), "normal", 1.0, "float32")
        out[p + "A_log"] = TensorDecl((self.heads,), "normal", 1.0, "float32")
        out[p + "D"] = TensorDecl((self.heads,), "one_plus_normal", 0.3, "float32")
        out[p + "norm"] = TensorDecl((self.inner,), "one_plus_normal", 0.1, "float32")
        return out

    def load(self, get: TensorGetter) -> None:
        p = self.prefix
        for lin in (self.proj, self.o_proj):
            lin.load(get)
            lin.prepare()
        self.conv_w, self.conv_b = get(p + "conv"), get(p + "conv.b")
        self.dt_bias, self.rate_log, self.skip, self.norm_w = get(p + "dt_bias"), get(p + "A_log"), get(p + "D"), get(p + "norm")

    def weight_tensors(self):
        return self.proj.tensors_kept() + self.o_proj.tensors_kept() + [
            self.conv_w, self.conv_b, self.dt_bias, self.rate_log, self.skip, self.norm_w]

    def library_products(self):
        return [(lin.weight, torch.float32) for lin in (self.proj, self.o_proj) if lin.weight is not None]

    def cache_need(self):
        return None

    def state_need(self):
        return StateNeed((self.heads * self.N * self.vdim + (self.taps - 1) * self.conv_channels,), "float32")

    def input_linear(self) -> Linear:
        """The product this mixer applies to its input first (float32 out).  A part that runs it beside
        another mixer may fuse the two products and hand each its columns (``forward_projected``)."""
        return self.proj

    def forward(self, h, ctx, cache):
        return self.forward_projected(self.proj(h, out_dtype=torch.float32), ctx, cache)

    def forward_projected(self, proj, ctx, cache):
        """``proj`` float32 [T, z | x | B | C | dt]; rows may be strided."""
        inner, GN, H = self.inner, self.groups * self.N, self.heads
        z, steps = proj[:, :inner], proj[:, 2 * inner + 2 * GN:]
        xbc = kernels.causal_conv(proj[:, inner:2 * inner + 2 * GN], self.conv_w, self.conv_b, ctx, cache.state,
                                  H * self.N * self.vdim, act="silu")
        x, B, C = xbc[:, :inner], xbc[:, inner:inner + GN], xbc[:, inner + GN:]
        y = kernels.linear_recurrence(C, B, x, ctx, cache.state, H, self.N, self.vdim, steps=steps, rate_log=self.rate_log,
                                      step_bias=self.dt_bias, skip=self.skip, share=H // self.groups)
        y = kernels.gated_group_norm(y, self.norm_w, z, inner // self.norm_groups, self.eps, "silu_first", self.dtype)
        return self.o_proj(y, out_dtype=torch.float32)


@register_mixer("rglru")
class RealGatedLRU(Part):
    """The recurrent block of Griffin (De et al., "Griffin: Mixing Gated Linear Recurrences with Local
    Attention for Efficient Language Models") around its real-gated linear recurrent unit.  Parameters:
    ``width`` of the two branches, ``blocks`` (the gates' matrices are block-diagonal), ``conv`` (taps),
    ``c`` (the factor in ln a = -c r softplus(lam)).  y = gelu_tanh(W_y h + b),  u = conv(W_x h + b);  in
    each block r = sigmoid(ra u + b), i = sigmoid(ri u + b);  a = exp(-c r softplus(lam)),
    S_t = a S_(t-1) + sqrt(1 - a^2) i u  from S = 0, the first token like every other;  result W_o (S * y).
    The request's slot keeps S [width] and, behind it, the convolution's last ``conv`` - 1 inputs.  The
    gates and everything behind them are float32 whatever the engine's dtype.  Tensors under the prefix:
    y, y.b, x, x.b, conv, conv.b, ra, ra.b, ri, ri.b, lam, o."""

    def __init__(self, hidden_size, prefix, dtype, device, width: int, blocks: int, conv: int, c: float = 8.0):
        super().__init__(hidden_size, prefix, dtype, device)
        self.width, self.blocks, self.taps, self.c = int(width), int(blocks), int(conv), float(c)
        if self.blocks <= 0 or self.width % self.blocks:
            raise ValueError(f"{prefix}: a width of {width} does not split into {blocks} blocks")
        if not 1 <= self.taps <= kernels.CONV_MAX_TAPS:
            raise ValueError(f"{prefix}: a convolution of {conv} taps is not served (1 to {kernels.CONV_MAX_TAPS})")
        mk = lambda s, n_in, n_out, b: Linear(prefix + s, n_in, n_out, b, weight_name=prefix + s, bias_name=prefix + s + ".b")
        self._branches = [mk("y", hidden_size, self.width, True), mk("x", hidden_size, self.width, True)]
        self.proj: Linear | None = None
        self.o_proj = mk("o", self.width, hidden_size, False)
        self.conv_w = self.conv_b = self.gates = self.bias_r = self.bias_i = self.lam = None

    def tensors(self):
        out = {}
        for lin in self._branches + [self.o_proj]:
            out.update(lin.tensors())
        p, bw = self.prefix, self.width // self.blocks
        out[p + "conv"] = TensorDecl((self.width, self.taps), "normal", 0.3, "float32")
        out[p + "conv.b"] = TensorDecl((self.width,), "normal", 0.1, "float32")
        for s in ("ra", "ri"):
            out[p + s] = TensorDecl((self.blocks, bw, bw), "normal", 0.2, "float32")
            out[p + s + ".b"] = TensorDecl((self.blocks, bw), "normal", 0.5, "float32")
        out[p + "lam"] = TensorDecl((self.width,), "normal", 1.0, "float32")
        return out

    def load(self, get: TensorGetter) -> None:
        p = self.prefix
        for lin in self._branches:
            lin.load(get)
        self.proj = fuse_linears(p + "yx", self._branches)
        for lin in self._branches:
            lin.weight = lin.bias = None
        self.o_proj.load(get)
        self.o_proj.prepare()
        self.conv_w, self.conv_b = get(p + "conv"), get(p + "conv.b")
        # both gates of a block as one matrix [2 bw, bw]: one batched product gives [T, blocks, r | i]
        self.gates = torch.cat([get(p + "ra"), get(p + "ri")], dim=1).contiguous()
        bw = self.width // self.blocks
        self.bias_r, self.bias_i = get(p + "ra.b").reshape(-1).contiguous(), get(p + "ri.b").reshape(-1).contiguous()
        self.lam = get(p + "lam")
        assert tuple(self.gates.shape) == (self.blocks, 2 * bw, bw)

    def weight_tensors(self):
        return self.proj.tensors_kept() + self.o_proj.tensors_kept() + [
            self.conv_w, self.conv_b, self.gates, self.bias_r, self.bias_i, self.lam]

    def library_products(self):
        return [(self.proj.weight, torch.float32), (self.o_proj.weight, torch.float32)]

    def cache_need(self):
        return None

    def state_need(self):
        return StateNeed((self.width + (self.taps - 1) * self.width,), "float32")

    def forward(self, h, ctx, cache):
        W, nb = self.width, self.blocks
        bw = W // nb
        T = h.shape[0]
        proj = self.proj(h, out_dtype=torch.float32)                       # [y | x] with their biases
        u = kernels.causal_conv(proj[:, W:], self.conv_w, self.conv_b, ctx, cache.state, W)
        g = torch.empty(T, nb, 2 * bw, dtype=torch.float32, device=h.device)
        kernels.batched_linear(u.view(T, nb, bw), self.gates, g)
        o = kernels.gated_scan(g, self.bias_r, self.bias_i, u, proj[:, :W], self.lam, self.c, ctx, cache.state, 0, self.dtype)
        return self.o_proj(o, out_dtype=torch.float32)


@register_mixer("gated_delta")
class GatedDeltaRule(Part):
    """The mixer of Gated DeltaNet (Yang, Kautz and Hatamizadeh, "Gated Delta Networks: Improving Mamba2 with Delta Rule").
    Parameters: ``heads`` (value heads), ``kv_heads`` (query/key heads; value head h reads number ``h // (heads /
    kv_heads)``), ``dim`` (query/key size), ``vdim``, ``conv`` (taps), ``eps`` of the output norm, ``unit_eps`` inside the
    root of the unit vectors' length.  Per token t: q, k and v leave their projections through a causal convolution per
    channel and SiLU; each head of q and k is scaled to length one, q besides by ``dim^(-1/2)``; every value head has a write
    strength beta_t = sigmoid(b_t) and a decay g_t = exp(-exp(A_log) softplus(a_t + dt_bias)), b_t and a_t from the input;

        w_t = beta_t (v_t - g_t S_(t-1)^T k_t),   S_t = g_t S_(t-1) + k_t w_t^T,   o_t = S_t^T q_t;

    o_t of a head is RMS-normed with ``norm`` [vdim], the same for all heads, gated by SiLU of a projection ``g`` of the input
    and projected.  The request's slot keeps S of every head (transposed, [heads, vdim, dim]) and, behind it, the
    convolutions' last ``conv`` - 1 inputs.  Everything
    between the projections and the output norm's result is float32 whatever the engine's dtype.  Tensors under the
    prefix: q, q.conv, k, k.conv, v, v.conv, b, a, A_log, dt_bias, g, norm, o."""

    def __init__(self, hidden_size, prefix, dtype, device, heads: int, kv_heads: int, dim: int, vdim: int, conv: int,
                 eps: float = 1e-6, unit_eps: float = 1e-6):
        super().__init__(hidden_size, prefix, dtype, device)
        self.heads, self.kv_heads, self.dim, self.vdim = int(heads), int(kv_heads), int(dim), int(vdim)
        self.taps, self.eps, self.unit_eps = int(conv), float(eps), float(unit_eps)
        if min(self.heads, self.kv_heads, self.dim, self.vdim) <= 0 or self.heads % self.kv_heads:
            raise ValueError(f"{prefix}: {heads} value heads of {vdim} do not share {kv_heads} query/key heads of {dim}")
        if not kernels.delta_takes_key_dim(self.dim):
            raise ValueError(f"{prefix}: a key size of {dim} per head is not served: the delta rule kernels take up to 256")
        if not 1 <= self.taps <= kernels.CONV_MAX_TAPS:
            raise ValueError(f"{prefix}: a convolution of {conv} taps is not served (1 to {kernels.CONV_MAX_TAPS})")
        self.qk, self.vs = self.kv_heads * self.dim, self.heads * self.vdim
        self.conv_channels = 2 * self.qk + self.vs
        mk = lambda s, n_in, n_out: Linear(prefix + s, n_in, n_out, False, weight_name=prefix + s)
        self._parts = [mk("q", hidden_size, self.qk), mk("k", hidden_size, self.qk), mk("v", hidden_size, self.vs),
                       mk("g", hidden_size, self.vs), mk("b", hidden_size, self.heads), mk("a", hidden_size, self.heads)]
        self.proj: Linear | None = None
        self.o_proj = mk("o", self.vs, hidden_size)
        self.conv_w = self.rate_log = self.dt_bias = self.norm_w = None

    def tensors(self):
        out = {}
        for lin in self._parts + [self.o_proj]:
            out.update(lin.tensors())
        p = self.prefix
        for s, n in (("q", self.qk), ("k", self.qk), ("v", self.vs)):
            out[f"{p}{s}.conv"] = TensorDecl((n, self.taps), "normal", 0.4, "float32")
        out[p + "A_log"] = TensorDecl((self.heads,), "normal", 1.0, "float32")
        out[p + "dt_bias"] = TensorDecl((self.heads,), "normal", 1.0, "float32")
        out[p + "norm"] = TensorDecl((self.vdim,), "one_plus_normal", 0.1, "float32")
        return out

    def load(self, get: TensorGetter) -> None:
        p = self.prefix
        for lin in self._parts + [self.o_proj]:
            lin.load(get)
        parts = list(self._parts)
        spare = -sum(lin.out_features for lin in parts) % 8
        if spare:                                  # rows of zeros at the end: the product's rows start at 16-byte borders
            pad = Linear(p + "pad", self.hidden_size, spare, False)
            pad.weight = parts[0].weight.new_zeros(spare, self.hidden_size)
            parts.append(pad)
        self.proj = fuse_linears(p + "qkvgba", parts)
        for lin in self._parts:
            lin.weight = None
        self.o_proj.prepare()
        # a tap's weights for all channels in a row
        self.conv_w = torch.cat([get(f"{p}{s}.conv") for s in "qkv"]).t().contiguous()
        self.rate_log, self.dt_bias = get(p + "A_log"), get(p + "dt_bias")
        self.norm_w = get(p + "norm").repeat(self.heads).contiguous()

    def weight_tensors(self):
        return self.proj.tensors_kept() + self.o_proj.tensors_kept() + [self.conv_w, self.rate_log, self.dt_bias, self.norm_w]

    def library_products(self):
        return [(lin.weight, torch.float32) for lin in (self.proj, self.o_proj) if lin is not None and lin.weight is not None]

    def cache_need(self):
        return None

    def state_need(self):
        return StateNeed((self.vs * self.dim + (self.taps - 1) * self.conv_channels,), "float32")

    step_vectors = staticmethod(kernels.chunk_vectors)

    def input_linear(self) -> Linear:
        return self.proj

    keeps_share_sums = True

    def forward(self, h, ctx, cache, keep_shares: bool = False):
        return self.forward_projected(self.proj(h, out_dtype=torch.float32), ctx, cache, keep_shares)

    def forward_projected(self, proj, ctx, cache, keep_shares: bool = False):
        """``proj`` float32 [T, q | k | v | g | b | a (| padding)]; rows may be strided."""
        H, C, vs = self.heads, self.conv_channels, self.vs
        qkv = kernels.conv_unit(proj[:, :C], self.conv_w, ctx, cache.state, vs * self.dim, self.dim, 2 * self.kv_heads,
                                self.kv_heads, self.dim ** -0.5, self.unit_eps)
        gate, b, a = proj[:, C:C + vs], proj[:, C + vs:C + vs + H], proj[:, C + vs + H:C + vs + 2 * H]
        o = kernels.delta_rule(qkv[:, :self.qk], qkv[:, self.qk:2 * self.qk], qkv[:, 2 * self.qk:], b, a, self.rate_log,
                               self.dt_bias, ctx, cache.state, H, self.dim, self.vdim, share=H // self.kv_heads,
                               chunks=kernels.step_chunks(ctx))
        y = kernels.gated_group_norm(o, self.norm_w, gate, self.vdim, self.eps, "silu", self.dtype)
        return self.o_proj(y, out_dtype=torch.float32, keep_shares=keep_shares)


@register_mixer("selective_scan")
class SelectiveScan(Part):
    """The mixer of Mamba (Gu and Dao, "Mamba: Linear-Time Sequence Modeling with Selective State Spaces").  Parameters:
    ``inner`` (channels), ``state`` (N states per channel), ``dt_rank``, ``conv`` (taps).  One projection of the input gives x
    and the gate z; a causal convolution per channel (with bias) and SiLU make the x that a second projection turns into a
    low-rank step, B and C (N each); the step passes ``dt`` (with bias) and softplus.  With vectors over a channel's states
    and A = -exp(A_log),

        S_t = exp(dt_t A) S_(t-1) + (dt_t x_t) B_t,   y_t = (C_t . S_t + D x_t) silu(z_t),

    and y is projected.  The request's slot keeps S ([N, inner]) and, behind it,
    the convolution's last ``conv`` - 1 inputs.  Projections and the convolution leave x in the engine's dtype; the steps,
    the decays, the state and the gate are float32.  Tensors under the prefix: in, conv, conv.b, x, dt, dt.b, A_log, D, o."""

    def __init__(self, hidden_size, prefix, dtype, device, inner: int, state: int, dt_rank: int, conv: int):
        super().__init__(hidden_size, prefix, dtype, device)
        self.inner, self.N, self.rank, self.taps = int(inner), int(state), int(dt_rank), int(conv)
        if min(self.inner, self.N, self.rank) <= 0 or self.N > kernels.SELECTIVE_SCAN_MAX_STATE:
            raise ValueError(f"{prefix}: {inner} channels of {state} states are not served (up to {kernels.SELECTIVE_SCAN_MAX_STATE} states)")
        if not 1 <= self.taps <= kernels.CONV_MAX_TAPS:
            raise ValueError(f"{prefix}: a convolution of {conv} taps is not served (1 to {kernels.CONV_MAX_TAPS})")
        mk = lambda s, n_in, n_out: Linear(prefix + s, n_in, n_out, False, weight_name=prefix + s)
        self.proj = mk("in", hidden_size, 2 * self.inner)
        self.x_proj = mk("x", self.inner, self.rank + 2 * self.N)
        self.dt_proj = mk("dt", self.rank, self.inner)
        self.o_proj = mk("o", self.inner, hidden_size)
        self.conv_w = self.conv_b = self.dt_bias = self.a2 = self.skip = None

    def _linears(self):
        return [self.proj, self.x_proj, self.dt_proj, self.o_proj]

    def tensors(self):
        out = {}
        for lin in self._linears():
            out.update(lin.tensors())
        p = self.prefix
        out[p + "conv"] = TensorDecl((self.inner, self.taps), "normal", 0.4, "float32")
        out[p + "conv.b"] = TensorDecl((self.inner,), "normal", 0.1, "float32")
        out[p + "dt.b"] = TensorDecl((self.inner,), "normal", 1.0, "float32")
        out[p + "A_log"] = TensorDecl((self.inner, self.N), "normal", 1.0, "float32")
        out[p + "D"] = TensorDecl((self.inner,), "one_plus_normal", 0.3, "float32")
        return out

    def load(self, get: TensorGetter) -> None:
        p = self.prefix
        for lin in self._linears():
            lin.load(get)
            lin.prepare()
        self.conv_w = get(p + "conv").t().contiguous()              # a tap's weights for all channels in a row
        self.conv_b, self.dt_bias, self.skip = get(p + "conv.b"), get(p + "dt.b"), get(p + "D")
        # the scan takes powers of two: A log2(e), a state's values for all channels in a row
        self.a2 = (-torch.exp(get(p + "A_log").double()) * math.log2(math.e)).t().to(torch.float32).contiguous()

    def weight_tensors(self):
        return [t for lin in self._linears() for t in lin.tensors_kept()] + [self.conv_w, self.conv_b, self.dt_bias, self.a2, self.skip]

    def library_products(self):
        return [(lin.weight, torch.float32) for lin in self._linears() if lin.weight is not None]

    def cache_need(self):
        return None

    def state_need(self):
        return StateNeed((self.N * self.inner + (self.taps - 1) * self.inner,), "float32")

    step_vectors = staticmethod(kernels.chunk_vectors)

    def input_linear(self) -> Linear:
        return self.proj

    keeps_share_sums = True

    def forward(self, h, ctx, cache, keep_shares: bool = False):
        return self.forward_projected(self.proj(h, out_dtype=torch.float32), ctx, cache, keep_shares)

    def forward_projected(self, proj, ctx, cache, keep_shares: bool = False):
        """``proj`` float32 [T, x | z]; rows may be strided."""
        f32 = torch.float32
        x = kernels.conv_unit(proj[:, :self.inner], self.conv_w, ctx, cache.state, self.N * self.inner, 256, 0, 0, bias=self.conv_b,
                              out_dtype=self.dtype)
        low = self.x_proj(x, out_dtype=f32)
        dt_in = low[:, :self.rank] if self.dtype == f32 else kernels.cast_rows(low[:, :self.rank], self.dtype)
        dt = self.dt_proj(dt_in, out_dtype=f32)
        y = kernels.selective_scan(dt, self.dt_bias, x, proj[:, self.inner:2 * self.inner], low[:, self.rank:], self.a2, self.skip,
                                   ctx, cache.state, 0, chunks=kernels.step_chunks(ctx))
        return self.o_proj(y, out_dtype=f32, keep_shares=keep_shares)


@register_mixer("matrix_lstm")
class MatrixLSTM(Part):
    """The matrix memory of xLSTM (mLSTM; Beck et al., "xLSTM: Extended Long Short-Term Memory").  Parameters: ``heads``, ``dim``
    (query/key size), ``vdim``, ``gate_cap``, ``eps`` of the output norm, ``floor`` (added to the denominator).  Per head, with
    q scaled by ``dim^(-1/2)`` and the cap bending both gates' logits:

        i_t = cap tanh((W_i h + b_i) / cap),  f_t = ln sigmoid(cap tanh((W_f h + b_f) / cap)),  m_t = max(f_t + m_(t-1), i_t),
        S_t = exp(f_t + m_(t-1) - m_t) S_(t-1) + exp(i_t - m_t) k_t v_t^T,   n_t likewise with k_t alone,
        o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + floor),

    S, n and m zero at the start.  The heads' outputs are RMS-normed one by one, scaled per channel by ``norm``, gated by the sigmoid
    of a projection ``g`` of the input and projected.  The request's slot keeps S, n and m of every head.  Everything between the
    projections and the output norm's result is float32 whatever the engine's dtype.  Tensors under the prefix: q, k, v, i, i.b, f, f.b, g,
    norm, o."""

    def __init__(self, hidden_size, prefix, dtype, device, heads: int, dim: int, vdim: int, gate_cap: float, eps: float = 1e-6,
                 floor: float = 1e-6):
        super().__init__(hidden_size, prefix, dtype, device)
        self.heads, self.dim, self.vdim = int(heads), int(dim), int(vdim)
        self.cap, self.eps, self.floor = float(gate_cap), float(eps), float(floor)
        if min(self.heads, self.dim, self.vdim) <= 0 or self.dim > kernels.MATRIX_LSTM_MAX_KEY:
            raise ValueError(f"{prefix}: {heads} heads of {dim} x {vdim} are not served (key sizes up to {kernels.MATRIX_LSTM_MAX_KEY})")
        if self.cap <= 0.0:
            raise ValueError(f"{prefix}: the gates' cap {gate_cap} must be positive")
        self.qk, self.vs = self.heads * self.dim, self.heads * self.vdim
        mk = lambda s, n_in, n_out: Linear(prefix + s, n_in, n_out, False, weight_name=prefix + s)
        self._parts = [mk("q", hidden_size, self.qk), mk("k", hidden_size, self.qk), mk("v", hidden_size, self.vs),
                       mk("g", hidden_size, self.vs), mk("i", hidden_size, self.heads), mk("f", hidden_size, self.heads)]
        self.proj: Linear | None = None
        self.o_proj = mk("o", self.vs, hidden_size)
        self.bias_in = self.bias_forget = self.norm_w = None

    def tensors(self):
        out = {}
        for lin in self._parts + [self.o_proj]:
            out.update(lin.tensors())
        p = self.prefix
        out[p + "i.b"] = TensorDecl((self.heads,), "normal", 1.0, "float32")
        out[p + "f.b"] = TensorDecl((self.heads,), "normal", 1.0, "float32")
        out[p + "norm"] = TensorDecl((self.vs,), "one_plus_normal", 0.1, "float32")
        return out

    def load(self, get: TensorGetter) -> None:
        p = self.prefix
        for lin in self._parts + [self.o_proj]:
            lin.load(get)
        parts = list(self._parts)
        spare = -sum(lin.out_features for lin in parts) % 8
        if spare:                                  # rows of zeros at the end: the product's rows start at 16-byte borders
            pad = Linear(p + "pad", self.hidden_size, spare, False)
            pad.weight = parts[0].weight.new_zeros(spare, self.hidden_size)
            parts.append(pad)
        self.proj = fuse_linears(p + "qkvgif", parts)
        for lin in self._parts:
            lin.weight = None
        self.o_proj.prepare()
        self.bias_in, self.bias_forget, self.norm_w = get(p + "i.b"), get(p + "f.b"), get(p + "norm")

    def weight_tensors(self):
        return self.proj.tensors_kept() + self.o_proj.tensors_kept() + [self.bias_in, self.bias_forget, self.norm_w]

    def library_products(self):
        return [(lin.weight, torch.float32) for lin in (self.proj, self.o_proj) if lin is not None and lin.weight is not None]

    def cache_need(self):
        return None

    def state_need(self):
        return StateNeed((kernels.matrix_lstm_state(self.heads, self.dim, self.vdim),), "float32")

    step_vectors = staticmethod(kernels.chunk_vectors)

    def input_linear(self) -> Linear:
        return self.proj

    keeps_share_sums = True

    def forward(self, h, ctx, cache, keep_shares: bool = False):
        return self.forward_projected(self.proj(h, out_dtype=torch.float32), ctx, cache, keep_shares)

    def forward_projected(self, proj, ctx, cache, keep_shares: bool = False):
        """``proj`` float32 [T, q | k | v | g | i | f (| padding)]; rows may be strided."""
        H, qk, vs = self.heads, self.qk, self.vs
        at = 2 * qk + 2 * vs
        o = kernels.matrix_lstm(proj[:, :qk], proj[:, qk:2 * qk], proj[:, 2 * qk:2 * qk + vs], proj[:, at:at + H], proj[:, at + H:at + 2 * H],
                                self.bias_in, self.bias_forget, self.cap, ctx, cache.state, H, self.dim, self.vdim,
                                q_scale=self.dim ** -0.5, floor=self.floor, chunks=kernels.step_chunks(ctx))
        y = kernels.gated_group_norm(o, self.norm_w, proj[:, 2 * qk + vs:at], self.vdim, self.eps, "sigmoid", self.dtype)
        return self.o_proj(y, out_dtype=torch.float32, keep_shares=keep_shares)
