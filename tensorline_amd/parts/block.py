"""Arrangements of a layer's parts.

What a model asks of a block (any class registered with ``@register_block``, built as
``cls(layer_spec, hidden_size, dtype, device)``):

* ``parts()``: the parts it is made of (for tensor declarations, loading, byte counts);
* ``cache_need()`` / ``state_need()``: what its mixer keeps per token and per request, or None;
* ``forward(x, carry, ctx, cache) -> carry``: updates the float32 residual stream ``x`` in place.
  ``carry`` is what the block before left to be added (a tensor, or None for the first block);
  what it returns is what is left for whoever runs next to add.
* optionally ``intake() -> Intake``: what else it can take as ``carry`` in place of a tensor.  A
  block that has it is also called with ``after=``, the intake of whoever runs next, and may
  return a carry in one of the forms that intake allows.  A block without it is only ever handed
  plain tensors and its successor only ever gets one from it.

``prenorm`` is the residual order of the reference (tensorline/paged.py:243-247,275-276):

    x <- x + carry;  h1 = norm1(x);  x <- x + mixer(h1);  h2 = norm2(x);  carry = ffn(h2)

The feed-forward output is not added at once: it is folded into the next block's (or the final
norm's) fused add-and-norm.

Few-row bfloat16 steps (decoding) can do without norm kernels: when a norm is ``deferrable()`` and
the parts on both sides of it set ``defers_norm``, the product that ends the branch before the norm
adds into the residual and prepares the norm's input, and the product after it applies the
division (``tensorline_amd.ops.kernels.NormedRows``).  The carry is then that object; the intake
says for which norm the successor takes it.
"""
from __future__ import annotations

import torch

from tensorline_amd.ops import kernels
from tensorline_amd.parts.base import Part
from tensorline_amd.parts.registry import build_part, register_block
from tensorline_amd.parts.spec import Intake, LayerSpec, TensorDecl


@register_block("prenorm")
class PreNormBlock:
    def __init__(self, spec: LayerSpec, hidden_size: int, dtype, device):
        common = dict(hidden_size=hidden_size, dtype=dtype, device=device)
        self.spec = spec
        self.mixer_norm = build_part("norm", spec.mixer_norm, layer_prefix=spec.prefix, **common)
        self.mixer = build_part("mixer", spec.mixer, layer_prefix=spec.prefix, **common)
        self.feed_forward_norm = build_part("norm", spec.feed_forward_norm, layer_prefix=spec.prefix, **common)
        self.feed_forward = build_part("feed_forward", spec.feed_forward, layer_prefix=spec.prefix, **common)

    def parts(self) -> list[Part]:
        return [self.mixer_norm, self.mixer, self.feed_forward_norm, self.feed_forward]

    def cache_need(self):
        fn = getattr(self.mixer, "cache_need", None)
        return fn() if fn is not None else None

    def state_need(self):
        fn = getattr(self.mixer, "state_need", None)
        return fn() if fn is not None else None

    def intake(self) -> Intake:
        """This block's first norm as NormedRows, if that norm can be carried and the mixer applies
        it; a ShareSum, if that norm adds one."""
        carried = _deferrable(self.mixer_norm) if getattr(self.mixer, "defers_norm", False) else None
        return Intake(carried, bool(getattr(self.mixer_norm, "adds_share_sums", False)))

    def forward(self, x: torch.Tensor, carry, ctx, cache, after: Intake | None = None):
        """``carry``: a tensor or None, or one of the forms this block's ``intake()`` offers: a
        ShareSum for its first norm to add, or that norm's NormedRows (already added to ``x``).
        ``after``: the intake of whoever runs next."""
        after = after or Intake()
        defer = kernels.can_defer_norm(x.shape[0], self.mixer_norm.dtype)
        h = carry if isinstance(carry, kernels.NormedRows) else self.mixer_norm.forward(x, carry)
        sink = self._sink(defer, x, self.mixer, _deferrable(self.feed_forward_norm), self.feed_forward)
        if sink is not None:
            h = self.mixer.forward(h, ctx, cache, sink=sink)
        else:
            h = self.feed_forward_norm.forward(x, self.mixer.forward(h, ctx, cache))
        sink = self._sink(defer, x, self.feed_forward, after.normed_rows_for, None)
        if sink is not None:
            return self.feed_forward.forward(h, ctx, sink=sink)
        if after.share_sums and getattr(self.feed_forward, "keeps_share_sums", False):
            return self.feed_forward.forward(h, ctx, keep_shares=True)
        return self.feed_forward.forward(h, ctx)

    @staticmethod
    def _sink(allowed: bool, x, producer, carried_norm, consumer):
        """The sink for ``producer``'s last product when the norm after it (``carried_norm`` =
        (weight, eps), None: it cannot be carried) can ride on it and on ``consumer`` (None: whoever
        offered the norm vouches for the consumer)."""
        if not allowed or carried_norm is None or not getattr(producer, "defers_norm", False):
            return None
        if consumer is not None and not getattr(consumer, "defers_norm", False):
            return None
        return kernels.NormSink(x, carried_norm[0], carried_norm[1])


def _deferrable(norm):
    fn = getattr(norm, "deferrable", None)
    return fn() if fn is not None else None


@register_block("prenorm_token_input")
class PreNormTokenInputBlock:
    """Pre-norm order with two things the plain block does not have: the feed-forward (and its norm)
    may be absent, and a per-layer input from the token ids may follow it:

        x <- x + carry;  x <- x + mixer(norm1(x));  [x <- x + ffn(norm2(x))];  [carry = token_input(x)]

    What the last stage leaves is handed on, not added: the next block's first norm (or the final
    norm) adds it in its own pass.  Carries are plain float32 tensors; no norm rides on a product
    here, so any norm kind fits."""

    def __init__(self, spec: LayerSpec, hidden_size: int, dtype, device):
        common = dict(hidden_size=hidden_size, dtype=dtype, device=device)
        self.spec = spec
        self.mixer_norm = build_part("norm", spec.mixer_norm, layer_prefix=spec.prefix, **common)
        self.mixer = build_part("mixer", spec.mixer, layer_prefix=spec.prefix, **common)
        self.feed_forward_norm = self.feed_forward = self.token_input = None
        if spec.feed_forward is not None:
            self.feed_forward_norm = build_part("norm", spec.feed_forward_norm, layer_prefix=spec.prefix, **common)
            self.feed_forward = build_part("feed_forward", spec.feed_forward, layer_prefix=spec.prefix, **common)
        if spec.token_input is not None:
            self.token_input = build_part("token_input", spec.token_input, layer_prefix=spec.prefix, **common)

    def parts(self) -> list[Part]:
        return [p for p in (self.mixer_norm, self.mixer, self.feed_forward_norm, self.feed_forward, self.token_input)
                if p is not None]

    def cache_need(self):
        fn = getattr(self.mixer, "cache_need", None)
        return fn() if fn is not None else None

    def state_need(self):
        fn = getattr(self.mixer, "state_need", None)
        return fn() if fn is not None else None

    def forward(self, x: torch.Tensor, carry, ctx, cache):
        y = self.mixer.forward(self.mixer_norm.forward(x, carry), ctx, cache)
        if self.feed_forward is not None:
            y = self.feed_forward.forward(self.feed_forward_norm.forward(x, y), ctx)
        if self.token_input is not None:
            y = self.token_input.forward(x, y, ctx)
        return y


@register_block("sandwich")
class SandwichBlock:
    """Every branch is normed on both sides: its input by a pre-norm, its output by a second norm before it
    joins the stream with a factor ``m`` (``LayerSpec.branch_scale``):

        x <- x + m * post1(mixer(norm1(x)));  [x <- x + m * post2(ffn(norm2(x)))]

    The feed-forward with its two norms may be absent.  A branch's normed output is not added at once: it is
    handed on as :class:`tensorline_amd.ops.kernels.NormedBranch`, and the norm that reads the stream next (this
    block's second pre-norm, the next block's first, the final norm) norms it, adds it and norms the sum in one
    pass.  Where whoever runs next does not take that form (``after.normed_branch``), the block adds it itself
    and leaves nothing."""

    def __init__(self, spec: LayerSpec, hidden_size: int, dtype, device):
        common = dict(hidden_size=hidden_size, dtype=dtype, device=device)
        self.spec = spec
        self.scale = float(spec.branch_scale)
        if spec.mixer_post_norm is None or (spec.feed_forward is not None and spec.feed_forward_post_norm is None):
            raise ValueError(f"{spec.prefix}: a sandwich block needs a norm behind every branch")
        self.mixer_norm = build_part("norm", spec.mixer_norm, layer_prefix=spec.prefix, **common)
        self.mixer = build_part("mixer", spec.mixer, layer_prefix=spec.prefix, **common)
        self.mixer_post = build_part("norm", spec.mixer_post_norm, layer_prefix=spec.prefix, **common)
        self.feed_forward_norm = self.feed_forward = self.feed_forward_post = None
        if spec.feed_forward is not None:
            self.feed_forward_norm = build_part("norm", spec.feed_forward_norm, layer_prefix=spec.prefix, **common)
            self.feed_forward = build_part("feed_forward", spec.feed_forward, layer_prefix=spec.prefix, **common)
            self.feed_forward_post = build_part("norm", spec.feed_forward_post_norm, layer_prefix=spec.prefix, **common)
        for norm in (self.mixer_post, self.feed_forward_post):
            if norm is not None and not hasattr(norm, "as_branch"):
                raise ValueError(f"{spec.prefix}: the norm behind a branch must offer as_branch (an RMS norm does)")
        if self.feed_forward_norm is not None and not getattr(self.feed_forward_norm, "adds_normed_branch", False):
            raise ValueError(f"{spec.prefix}: the feed-forward's pre-norm must take a normed branch as its residual")

    def parts(self) -> list[Part]:
        return [p for p in (self.mixer_norm, self.mixer, self.mixer_post, self.feed_forward_norm, self.feed_forward,
                            self.feed_forward_post) if p is not None]

    def cache_need(self):
        fn = getattr(self.mixer, "cache_need", None)
        return fn() if fn is not None else None

    def state_need(self):
        fn = getattr(self.mixer, "state_need", None)
        return fn() if fn is not None else None

    def intake(self) -> Intake:
        return Intake(None, False, bool(getattr(self.mixer_norm, "adds_normed_branch", False)))

    def forward(self, x: torch.Tensor, carry, ctx, cache, after: Intake | None = None):
        y = self.mixer.forward(self.mixer_norm.forward(x, carry), ctx, cache)
        branch = self.mixer_post.as_branch(y, self.scale)
        if self.feed_forward is not None:
            y = self.feed_forward.forward(self.feed_forward_norm.forward(x, branch), ctx)
            branch = self.feed_forward_post.as_branch(y, self.scale)
        if after is not None and after.normed_branch:
            return branch
        kernels.add_normed_branch(x, branch)
        return None


@register_block("parallel_branches")
class ParallelBranchesBlock:
    """One norm ahead of both branches, which run side by side on its output and join the stream together:

        h = norm1(x);  x <- x + m * (mixer(h) + ffn(h))

    with the factor ``m`` = ``LayerSpec.branch_scale``; the feed-forward may be absent.  A mixer or feed-forward that sets
    ``keeps_share_sums`` may leave its last product in its shares of K.  The branches' outputs are not added at once:
    they are handed on as :class:`tensorline_amd.ops.kernels.ScaledBranches`, and the norm that reads the stream next adds
    both in its own pass.  Where whoever runs next does not take that form (``after.scaled_branches``), the block adds
    them itself and leaves nothing."""

    def __init__(self, spec: LayerSpec, hidden_size: int, dtype, device):
        common = dict(hidden_size=hidden_size, dtype=dtype, device=device)
        self.spec = spec
        self.scale = float(spec.branch_scale)
        if spec.feed_forward_norm is not None:
            raise ValueError(f"{spec.prefix}: both branches read the one norm: there is no norm for the feed-forward")
        self.norm = build_part("norm", spec.mixer_norm, layer_prefix=spec.prefix, **common)
        self.mixer = build_part("mixer", spec.mixer, layer_prefix=spec.prefix, **common)
        self.feed_forward = None
        if spec.feed_forward is not None:
            self.feed_forward = build_part("feed_forward", spec.feed_forward, layer_prefix=spec.prefix, **common)

    def parts(self) -> list[Part]:
        return [p for p in (self.norm, self.mixer, self.feed_forward) if p is not None]

    def cache_need(self):
        fn = getattr(self.mixer, "cache_need", None)
        return fn() if fn is not None else None

    def state_need(self):
        fn = getattr(self.mixer, "state_need", None)
        return fn() if fn is not None else None

    def intake(self) -> Intake:
        return Intake(scaled_branches=bool(getattr(self.norm, "adds_scaled_branches", False)))

    def forward(self, x: torch.Tensor, carry, ctx, cache, after: Intake | None = None):
        h = self.norm.forward(x, carry)
        shares = lambda part: {"keep_shares": True} if getattr(part, "keeps_share_sums", False) else {}
        y = self.mixer.forward(h, ctx, cache, **shares(self.mixer))
        ff = self.feed_forward
        branches = kernels.ScaledBranches(y, ff.forward(h, ctx, **shares(ff)) if ff is not None else None, self.scale)
        if after is not None and after.scaled_branches:
            return branches
        kernels.add_scaled_branches(x, branches)
        return None


class ChannelScale(Part):
    """A learned factor per channel on what a branch adds to the stream."""

    def __init__(self, hidden_size, prefix, dtype, device, name: str):
        super().__init__(hidden_size, prefix, dtype, device)
        self.name = prefix + name
        self.weight: torch.Tensor | None = None

    def tensors(self):
        return {self.name: TensorDecl((self.hidden_size,), "one_plus_normal", 0.2, "float32")}

    def load(self, get) -> None:
        self.weight = get(self.name)

    def weight_tensors(self):
        return [self.weight]


@register_block("parallel_normed_branches")
class ParallelNormedBranchesBlock:
    """Two branches side by side on the same stream, each behind an RMS norm of its own and with an optional learned factor per
    channel on its result (``LayerSpec.channel_scales``):

        x <- x + (s1 * mixer(norm1(x)) + s2 * ffn(norm2(x)))

    The feed-forward (with its norm and factor) may be absent.  Both norms divide by the same root mean square, so one kernel
    adds what the layer before left, and makes both inputs.  The branches' outputs are not added at once: they are handed on as
    :class:`tensorline_amd.ops.kernels.JoinedBranches` (the feed-forward's as its experts' rows where it can leave them so), and
    the norms that read the stream next add both in their own pass.  Where whoever runs next does not take that form
    (``after.joined_branches``), the block adds them itself and leaves nothing."""

    def __init__(self, spec: LayerSpec, hidden_size: int, dtype, device):
        common = dict(hidden_size=hidden_size, dtype=dtype, device=device)
        self.spec = spec
        self.dtype = dtype
        self.mixer_norm = build_part("norm", spec.mixer_norm, layer_prefix=spec.prefix, **common)
        self.mixer = build_part("mixer", spec.mixer, layer_prefix=spec.prefix, **common)
        self.feed_forward_norm = self.feed_forward = self.mixer_scale = self.feed_forward_scale = None
        scale = lambda i: ChannelScale(prefix=spec.prefix, name=spec.channel_scales[i], **common) if spec.channel_scales else None
        self.mixer_scale = scale(0)
        if spec.feed_forward is not None:
            self.feed_forward_norm = build_part("norm", spec.feed_forward_norm, layer_prefix=spec.prefix, **common)
            self.feed_forward = build_part("feed_forward", spec.feed_forward, layer_prefix=spec.prefix, **common)
            self.feed_forward_scale = scale(1)
        norms = [n for n in (self.mixer_norm, self.feed_forward_norm) if n is not None]
        if any(not getattr(n, "adds_joined_branches", False) for n in norms) or len({n.eps for n in norms}) != 1:
            raise ValueError(f"{spec.prefix}: both norms must be RMS norms of one eps: they share a root mean square")

    def parts(self) -> list[Part]:
        return [p for p in (self.mixer_norm, self.mixer, self.mixer_scale, self.feed_forward_norm, self.feed_forward,
                            self.feed_forward_scale) if p is not None]

    def cache_need(self):
        fn = getattr(self.mixer, "cache_need", None)
        return fn() if fn is not None else None

    def state_need(self):
        fn = getattr(self.mixer, "state_need", None)
        return fn() if fn is not None else None

    def intake(self) -> Intake:
        return Intake(joined_branches=True)

    def forward(self, x: torch.Tensor, carry, ctx, cache, after: Intake | None = None):
        ff = self.feed_forward
        h1, h2 = kernels.join_norms(x, carry, self.mixer_norm.weight, self.feed_forward_norm.weight if ff is not None else None,
                                    self.mixer_norm.eps, self.dtype)
        keep = lambda part, flag, kw: {kw: True} if getattr(part, flag, False) else {}
        weight = lambda scale: scale.weight if scale is not None else None
        y1 = self.mixer.forward(h1, ctx, cache, **keep(self.mixer, "keeps_share_sums", "keep_shares"))
        y2 = None
        if ff is not None:
            y2 = ff.forward(h2, ctx, **keep(ff, "keeps_share_sums", "keep_shares"), **keep(ff, "keeps_expert_rows", "keep_rows"))
        branches = kernels.JoinedBranches(y1, weight(self.mixer_scale), y2, weight(self.feed_forward_scale))
        if after is not None and after.joined_branches:
            return branches
        kernels.join_norms(x, branches, None, None, 0.0, None)
        return None
