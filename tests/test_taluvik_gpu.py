"""Taluvik on the GPU against the plain implementation (tests/plain_taluvik.py): every mechanism alone, whole
prompts, token-by-token decoding, portions, mixed batches with pages and slots used again, tokens made to stand out
at the places where a cache, a state or a chunk can lose them, long decoding, and greedy generation through the
entry point."""
import copy
import random

import numpy as np
import pytest
import torch

from tests import plain_taluvik as P
from tests.helpers import steps_portions, steps_prefill_then_decode, steps_whole
from tests.samovik_helpers import rel_error, run_steps
from tests.taluvik_helpers import (BANDS, CFG_A, CFG_B, CFG_C, CONFIGS, _attn, _delta, _mamba, build, one_layer, random_config,
                                   typed)
from tests.test_samovik_gpu import mixed_steps

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = ["float32", "bfloat16"]
LIMIT = {"float32": 3e-5, "bfloat16": 5e-2}          # of the logits' own root mean square


def tokens_for(cfg, n, seed):
    rng = random.Random(seed)
    return [rng.randrange(cfg["vocab"]) for _ in range(n)]


def run_and_check(model, steps, cfg, w, reqs, dtype, what="", **kw):
    """Run the steps and hold every position against the plain implementation."""
    got = run_steps(model, steps, **kw)
    for rid, toks in reqs.items():
        want = P.forward(cfg, w, toks).numpy()
        rows = got[rid]
        assert sorted(rows) == list(range(len(toks))), f"{what}: {rid} is missing positions"
        errs = {p: rel_error(rows[p], want[p]) for p in rows}
        first_bad = next((p for p in sorted(rows) if not errs[p] <= LIMIT[dtype]), None)
        assert first_bad is None, (f"{what} {dtype}: request {rid}: first wrong position {first_bad} of {len(toks)}, "
                                   f"worst error {max(errs.values()):.3e}")


def _session(model, page=16, blocks=64, slots=4):
    from tensorline_amd.cache.manager import CacheManager
    from tensorline_amd.engine.runner import ModelRunner
    cache = CacheManager(model.cache_needs(), model.schedule, model.state_needs(), page_size=page, num_blocks=blocks,
                         max_requests=slots, dtype=model.dtype, device=DEV, input_state_need=model.input_state_need())
    return cache, ModelRunner(model, cache)


def _step_context(cache, runner, portions):
    """``portions``: (request, first position, count).  Returns the step's context and cache views."""
    from tensorline_amd.engine.batch import StepEntry
    entries = []
    for rid, lo, n in portions:
        if not cache.has_request(rid):
            cache.add_request(rid)
        cache.grow(rid, lo + n)
        entries.append(StepEntry(rid, [0] * n, lo, [0]))
    packed = runner.pack(entries)
    return runner.context(packed, runner._upload(packed.data))


def _rms_error(got, want):
    return ((got - want).pow(2).mean().sqrt() / want.pow(2).mean().sqrt()).item()


class _Step:
    """A step's index data for kernels called on their own: sequences of ``lens`` tokens on state slots in reverse order."""

    def __init__(self, lens, chunked):
        from tensorline_amd.engine.batch import StepFacts
        i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=DEV)
        at = [0]
        for n in lens:
            at.append(at[-1] + n)
        self.num_seqs, self.q_start = len(lens), i32(at)
        self.seq_of_token = i32([s for s, n in enumerate(lens) for _ in range(n)])
        self.state_slots = i32(list(range(len(lens)))[::-1])
        self.facts = StepFacts(max_query_len=max(lens), decode_only=max(lens) == 1, num_seqs=len(lens), q_lens=list(lens),
                               starts=[0] * len(lens))
        self.chunks = None
        if chunked:
            from tensorline_amd.ops import kernels
            v = kernels.chunk_vectors(StepFacts(max_query_len=10 ** 6, num_seqs=len(lens), q_lens=list(lens)))
            if v["chunks.seq"]:
                self.chunks = kernels.SequenceChunks(*(i32(v["chunks." + n]) for n in ("seq", "row", "first")),
                                                     walked=min(lens) <= kernels.WALK_TOKENS)


# ---- every mechanism alone -------------------------------------------------------------------------
@pytest.mark.parametrize("H", [4, 96, 130, 1000, 4096, 5121])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_branches_join_the_stream_and_the_layer_norm_reads_it(H, dtype):
    from tensorline_amd.ops import kernels
    torch.manual_seed(H)
    T = 600 if H == 4096 else 7
    x, y1, y2 = torch.randn(T, H) + 3.0, torch.randn(T, H), torch.randn(T, H)
    w, b = torch.randn(H), torch.randn(H)
    tol = dict(atol=2e-5, rtol=2e-5) if dtype == torch.float32 else dict(atol=3e-2, rtol=1e-2)
    for branches, total in ((None, x.double()), (kernels.ScaledBranches(y1.to(DEV), y2.to(DEV), 0.35), x.double() + 0.35 * (y1.double() + y2.double())),
                            (kernels.ScaledBranches(y1.to(DEV), None, -2.0), x.double() - 2.0 * y1.double()), (y1.to(DEV), x.double() + y1.double()),
                            (kernels.ScaledBranches(kernels.ShareSum(torch.stack((y1, y2, x)).to(DEV)), kernels.ShareSum(torch.stack((y2, y2)).to(DEV)), 0.5),
                             x.double() * 1.5 + 0.5 * y1.double() + 1.5 * y2.double())):
        got_x = x.to(DEV).clone()
        got = kernels.add_layernorm(got_x, branches, w.to(DEV), b.to(DEV), 1e-5, dtype)
        torch.testing.assert_close(got_x.double().cpu(), total, atol=1e-5, rtol=1e-5)
        torch.testing.assert_close(got.double().cpu(), P.layer_norm(total, w.double(), b.double(), 1e-5), **tol)
        rows = torch.tensor([T - 1, 0, 2], dtype=torch.int32, device=DEV)
        got_x = x.to(DEV).clone()
        got = kernels.add_layernorm(got_x, branches, w.to(DEV), b.to(DEV), 1e-5, dtype, rows=rows)
        assert torch.equal(got_x.cpu(), x)
        torch.testing.assert_close(got.double().cpu(), P.layer_norm(total[rows.cpu().long()], w.double(), b.double(), 1e-5), **tol)
    got_x = x.to(DEV).clone()
    kernels.add_scaled_branches(got_x, kernels.ScaledBranches(y1.to(DEV), y2.to(DEV), 0.35))
    torch.testing.assert_close(got_x.double().cpu(), x.double() + 0.35 * (y1.double() + y2.double()), atol=1e-5, rtol=1e-5)


def test_layer_norm_keeps_its_digits_behind_a_large_mean():
    from tensorline_amd.ops import kernels
    torch.manual_seed(0)
    x = torch.randn(5, 512) + 1000.0
    one, zero = torch.ones(512), torch.zeros(512)
    got = kernels.add_layernorm(x.to(DEV).clone(), None, one.to(DEV), zero.to(DEV), 1e-6, torch.float32).double().cpu()
    torch.testing.assert_close(got, P.layer_norm(x.double(), one.double(), zero.double(), 1e-6), atol=2e-4, rtol=1e-4)


@pytest.mark.parametrize("case", [
    # query heads, key heads, dim, vdim, turned dims
    (4, 2, 24, 24, 8), (3, 1, 10, 7, 10), (2, 2, 128, 128, 32), (1, 1, 6, 6, 2), (5, 5, 250, 200, 250), (6, 2, 64, 32, 64), (2, 1, 16, 40, 0),
    (2, 1, 7, 9, 4)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_halves_turned_heads_normed_without_weights_and_the_cache_write(case, dtype):
    from tensorline_amd.ops import kernels
    from tensorline_amd.parts.rotary import band_frequencies
    H, G, d, dv, rot = case
    D = -(-max(d, dv) // 16) * 16
    T, page, pages = 23, 8, 9
    torch.manual_seed(sum(case))
    proj = torch.randn(T, (H + G) * d + G * dv + 3)
    pos = torch.randint(0, 100, (T,), dtype=torch.int32)
    slots = torch.randperm(pages * page)[:T].to(torch.int32)
    freq = band_frequencies(rot, 300.0, BANDS).to(DEV) if rot else None
    kc = torch.full((pages, page, G, D), 7.0).to(dtype).to(DEV)
    vc = torch.full((pages, G, D, page), 7.0).to(dtype).to(DEV)
    got_q = kernels.head_norm_rotate_store(proj.to(DEV), pos.to(DEV), None, None, 1e-5, freq, 1.0, kc, vc, slots.to(DEV), H, G, d, dv, False,
                                           dtype, plain_norm=True, halves=True)
    x = proj.double()
    q, k = x[:, :H * d].view(T, H, d), x[:, H * d:(H + G) * d].view(T, G, d)
    v = x[:, (H + G) * d:(H + G) * d + G * dv].view(T, G, dv)
    if rot:
        freqs = P.frequencies(rot, 300.0, BANDS)
        q, k = P.turn_halves(q, pos.tolist(), freqs), P.turn_halves(k, pos.tolist(), freqs)
    q, k = P.rms_scale(q, 1e-5), P.rms_scale(k, 1e-5)          # behind the rotation, as the design states it
    tol = dict(atol=2e-4, rtol=1e-4) if dtype == torch.float32 else dict(atol=3e-2, rtol=2e-2)
    got_q = got_q.double().cpu().view(T, H, D)
    torch.testing.assert_close(got_q[:, :, :d], q, **tol)
    got_k = kc.double().cpu().view(-1, G, D)[slots.long()]
    torch.testing.assert_close(got_k[:, :, :d], k, **tol)
    got_v = vc.double().cpu().permute(0, 3, 1, 2).reshape(-1, G, D)[slots.long()]
    torch.testing.assert_close(got_v[:, :, :dv], v, **tol)
    assert not got_q[:, :, d:].any() and not got_k[:, :, d:].any() and not got_v[:, :, dv:].any()


@pytest.mark.parametrize("lens", [[1, 1, 1], [37, 1, 64], [3, 200, 2], [1] * 70, [9]])
@pytest.mark.parametrize("case", [
    # unit, normed units, scaled units, further channels, taps
    (24, 4, 2, 160, 4), (7, 3, 1, 20, 3), (128, 2, 1, 128, 4), (64, 6, 3, 33, 1), (256, 2, 2, 0, 2), (4, 2, 1, 8, 7), (130, 2, 1, 5, 16)])
def test_convolution_into_unit_vectors(case, lens):
    """Two steps: the second starts from the inputs the first one kept; a slot of zeros is a sequence's beginning."""
    from tensorline_amd.ops import kernels
    unit, n_unit, n_scaled, more, taps = case
    C, off = unit * n_unit + more, 6
    torch.manual_seed(unit + len(lens))
    wt = torch.randn(C, taps)
    first = [1 + (5 * i) % 11 for i in range(len(lens))]
    xs = [torch.randn(a + b, C) for a, b in zip(first, lens)]
    state = torch.zeros(len(lens) + 1, off + (taps - 1) * C, device=DEV)
    outs = []
    for part, ls in ((0, first), (1, lens)):
        step = _Step(ls, False)
        flat = torch.cat([x[:a] if part == 0 else x[a:] for x, a in zip(xs, first)])
        wide = torch.cat((flat, torch.full((flat.shape[0], 5), 9.0)), 1).to(DEV)
        out = kernels.conv_unit(wide[:, :C], wt.t().contiguous().to(DEV), step, state, off, unit, n_unit, n_scaled, 0.3, 1e-6).double().cpu()
        at, rows = 0, []
        for n in ls:
            rows.append(out[at:at + n])
            at += n
        outs.append(rows)
    assert not state[:, :off].any() and not state[len(lens)].any()
    for i, x in enumerate(xs):
        want = P.silu(P.causal_conv(x.double(), wt.double()))
        heads = P.unit_rows(want[:, :unit * n_unit].view(-1, n_unit, unit))
        heads[:, :n_scaled] *= 0.3
        want[:, :unit * n_unit] = heads.reshape(-1, unit * n_unit)
        torch.testing.assert_close(torch.cat((outs[0][i], outs[1][i])), want, atol=2e-6, rtol=1e-5)


@pytest.mark.parametrize("C,taps", [(88, 4), (50, 6), (300, 1), (1024, 3), (7, 16)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_convolution_with_bias_and_without_units(C, taps, dtype):
    from tensorline_amd.ops import kernels
    torch.manual_seed(C)
    wt, bias = torch.randn(C, taps), torch.randn(C)
    lens = [70, 1, 33]
    xs = [torch.randn(n + 2, C) for n in lens]
    state = torch.zeros(4, (taps - 1) * C, device=DEV)
    outs = [[], [], []]
    for ls, lo in ((lens, 0), ([2, 2, 2], None), ):
        step = _Step(ls, False)
        flat = torch.cat([x[:n] if lo == 0 else x[n:] for x, n in zip(xs, lens)]).to(DEV)
        out = kernels.conv_unit(flat, wt.t().contiguous().to(DEV), step, state, 0, 256, 0, 0, bias=bias.to(DEV), out_dtype=dtype).double().cpu()
        at = 0
        for i, n in enumerate(ls):
            outs[i].append(out[at:at + n])
            at += n
    for i, x in enumerate(xs):
        want = P.silu(P.causal_conv(x.double(), wt.double(), bias.double()))
        torch.testing.assert_close(torch.cat(outs[i]), want, **(dict(atol=1e-5, rtol=1e-5) if dtype == torch.float32 else dict(atol=2e-2, rtol=1e-2)))


def _plain_delta(q, k, v, b, a, rate_log, bias, S):
    """One head: q, k [T, dk], v [T, dv]; returns (outputs, the state behind the last token)."""
    out = torch.zeros(v.shape, dtype=torch.float64)
    for t in range(q.shape[0]):
        S = S * torch.exp(-torch.exp(rate_log) * P.softplus(a[t] + bias))
        u = torch.sigmoid(b[t]) * (v[t] - S.T @ k[t])
        S = S + torch.outer(k[t], u)
        out[t] = S.T @ q[t]
    return out, S


@pytest.mark.parametrize("chunked", [False, True])
@pytest.mark.parametrize("lens", [[1, 1, 1], [150, 1, 64, 65], [63, 32, 33, 2], [300]])
@pytest.mark.parametrize("case", [
    # heads, share, dk, dv, what the decays are like
    (4, 2, 24, 40, "mixed"), (3, 3, 9, 13, "mixed"), (2, 1, 128, 64, "long"), (2, 2, 64, 128, "strong"), (1, 1, 16, 5, "none"), (2, 1, 96, 16, "mixed"),
    (2, 1, 130, 20, "mixed"), (6, 1, 32, 17, "jumps")])
def test_delta_rule_token_by_token_and_in_chunks(case, lens, chunked):
    """Two steps on one set of states, slots in another order than the sequences.  Decays from none at all to one that
    forgets everything at once between tokens that keep everything ("jumps"), which a chunk's sums of logarithms must
    not blur; keys repeat, so that what a key held has to be taken out again."""
    from tensorline_amd.ops import kernels
    H, share, dk, dv, kind = case
    torch.manual_seed(dk + dv + len(lens))
    G, off = H // share, 3
    T = sum(lens)
    state = torch.randn(len(lens) + 1, off + H * dk * dv) * 0.5
    dev_state = state.to(DEV).clone()
    rate_log, bias = torch.randn(H) * (0.5 if kind == "mixed" else 0.1), torch.randn(H)
    shift = {"mixed": -1.0, "long": -6.0, "strong": 4.0, "none": -40.0, "jumps": -5.0}[kind]
    plain_S = [[state[len(lens) - 1 - s, off:].view(H, dv, dk)[h].t().double() for h in range(H)] for s in range(len(lens))]
    for rep in range(2):
        q = P.unit_rows(torch.randn(T, G, dk).double()).float() * dk ** -0.5
        k = P.unit_rows(torch.randn(T, G, dk).double()).float()
        k[1::3] = k[:1]                                         # a third of the tokens write to one key
        v, b, a = torch.randn(T, H * dv), torch.randn(T, H) * 2, torch.randn(T, H) + shift
        if kind == "jumps":
            a[::7] = 90.0
        step = _Step(lens, chunked)
        wide = torch.cat((q.reshape(T, -1), k.reshape(T, -1), v, b, a, torch.zeros(T, 1)), 1).to(DEV)
        cuts = [0, G * dk, 2 * G * dk, 2 * G * dk + H * dv, 2 * G * dk + H * dv + H, 2 * G * dk + H * dv + 2 * H]
        piece = [wide[:, cuts[i]:cuts[i + 1]] for i in range(5)]
        got = kernels.delta_rule(*piece, rate_log.to(DEV), bias.to(DEV), step, dev_state, H, dk, dv, share=share, state_offset=off,
                                 chunks=step.chunks).double().cpu().view(T, H, dv)
        at = 0
        for s, n in enumerate(lens):
            for h in range(H):
                want, plain_S[s][h] = _plain_delta(q[at:at + n, h // share].double(), k[at:at + n, h // share].double(),
                                                   v[at:at + n].view(n, H, dv)[:, h].double(), b[at:at + n, h].double(), a[at:at + n, h].double(),
                                                   rate_log[h].double(), bias[h].double(), plain_S[s][h])
                err = _rms_error(got[at:at + n, h], want)
                assert err < 3e-6, f"step {rep}, sequence {s} of {n}, head {h}: {err:.2e}"
                kept = dev_state[len(lens) - 1 - s, off:].view(H, dv, dk)[h].t().double().cpu()
                assert _rms_error(kept, plain_S[s][h]) < 3e-6
            at += n
    assert torch.equal(dev_state[:, :off].cpu(), state[:, :off]) and torch.equal(dev_state[len(lens)].cpu(), state[len(lens)])


@pytest.mark.parametrize("chunked", [False, True])
@pytest.mark.parametrize("lens", [[1, 1, 1], [150, 1, 64, 65], [63, 32, 33, 2], [700]])
@pytest.mark.parametrize("inner,N", [(88, 12), (50, 1), (300, 16), (33, 17), (70, 40), (20, 256), (17, 8), (130, 100)])
def test_selective_scan_token_by_token_and_in_chunks(inner, N, lens, chunked):
    from tensorline_amd.ops import kernels
    torch.manual_seed(inner + N)
    T, off = sum(lens), 5
    state = torch.randn(len(lens) + 1, off + N * inner)
    dev_state = state.to(DEV).clone()
    A, D, bias = -torch.exp(torch.randn(inner, N)), torch.randn(inner), torch.randn(inner) - 3.0
    a2 = (A.double() / np.log(2.0)).t().float().contiguous()
    S = [state[len(lens) - 1 - s, off:].view(N, inner).t().double() for s in range(len(lens))]
    for rep in range(2):
        dt, x, z, bc = torch.randn(T, inner) * 2, torch.randn(T, inner), torch.randn(T, inner), torch.randn(T, 2 * N)
        step = _Step(lens, chunked)
        wide = torch.cat((torch.zeros(T, 3), z, bc), 1).to(DEV)
        got = kernels.selective_scan(dt.to(DEV), bias.to(DEV), x.to(DEV), wide[:, 3:3 + inner], wide[:, 3 + inner:], a2.to(DEV), D.to(DEV),
                                     step, dev_state, off, chunks=step.chunks).double().cpu()
        at = 0
        for s, n in enumerate(lens):
            want = torch.zeros(n, inner, dtype=torch.float64)
            for t in range(n):
                step_dt, xt = P.softplus(dt[at + t].double() + bias.double()), x[at + t].double()
                S[s] = torch.exp(step_dt[:, None] * A.double()) * S[s] + (step_dt * xt)[:, None] * bc[at + t, :N].double()[None]
                want[t] = S[s] @ bc[at + t, N:].double() + D.double() * xt
            want *= P.silu(z[at:at + n].double())
            assert _rms_error(got[at:at + n], want) < 3e-6, f"step {rep}, sequence {s} of {n}"
            assert _rms_error(dev_state[len(lens) - 1 - s, off:].view(N, inner).t().double().cpu(), S[s]) < 3e-6
            at += n
    assert torch.equal(dev_state[:, :off].cpu(), state[:, :off]) and torch.equal(dev_state[len(lens)].cpu(), state[len(lens)])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,ff", [(88, 136), (88, 7), (320, 1024), (1024, 640)])
def test_feed_forward_alone(width, ff, dtype):
    """From one row to many: the few-row and the mid-row product with the gate in their epilogues, with and without K cut
    into shares, and the product with a pass of its own behind it."""
    cfg = one_layer("mamba1", _mamba(8, 1, 1, 1), ff, width=width)
    model, w = build(cfg, dtype, seed=3)
    W = P.as_double(w)
    for rows in (1, 5, 17, 33, 64, 65, 300):
        torch.manual_seed(rows)
        h = torch.randn(rows, width).to(torch.bfloat16).float()
        got = model.blocks[0].feed_forward.forward(h.to(DEV).to(model.dtype), None).float().cpu()
        err = _rms_error(got, P.gated_ff(h.double(), W, "l0.mlp.").float())
        assert err < (1e-5 if dtype == "float32" else 1e-2), f"{rows} rows: {err:.3e}"


MIXERS = [
    ("attention", _attn(4, 2, 24, 40, 19, 8)), ("attention", _attn(1, 1, 10, 7, 16, 10, scaling=None, softcap=None)),
    ("attention", _attn(6, 1, 64, 40, 50, 32, softcap=2.0)), ("attention", _attn(2, 2, 128, 96, 0, 128, scale=0.05)),
    ("attention", _attn(9, 3, 32, 32, 1, 16)), ("attention", _attn(18, 2, 32, 16, 200, 0)), ("attention", _attn(2, 1, 5, 3, 2, 4)),
    ("delta", _delta(4, 2, 24, 40)), ("delta", _delta(3, 1, 9, 13, 1)), ("delta", _delta(1, 1, 128, 64, 6)), ("delta", _delta(5, 5, 16, 7, 2)),
    ("delta", _delta(2, 1, 200, 24, 3)), ("delta", _delta(8, 2, 64, 128)),
    ("mamba1", _mamba(88, 12, 8)), ("mamba1", _mamba(50, 1, 1, 6)), ("mamba1", _mamba(144, 40, 16, 1)), ("mamba1", _mamba(24, 20, 5, 2)),
    ("mamba1", _mamba(256, 16, 24, 16)),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", range(len(MIXERS)))
def test_mixer_alone(case, dtype):
    """Three sequences in one batch, each from its first token, then each continued by a second step of other
    sizes (one token among them): the mixer's outputs against the plain ones of the whole sequences."""
    kind, mixer = MIXERS[case]
    cfg = one_layer(kind, mixer, width=72)
    model, w = build(cfg, dtype, seed=case)
    W = P.as_double(w)
    first, second = [37, 1, 150], [1, 20, 3]
    torch.manual_seed(case)
    hs = [torch.randn(a + b, 72).to(torch.bfloat16).float() for a, b in zip(first, second)]
    cache, runner = _session(model)
    mix = model.blocks[0].mixer
    ctx, views = _step_context(cache, runner, [(i, 0, n) for i, n in enumerate(first)])
    got1 = mix.forward(torch.cat([h[:n] for h, n in zip(hs, first)]).to(DEV).to(model.dtype), ctx, views[0]).float().cpu()
    for i, n in enumerate(first):
        cache.trim(i, n)
    ctx, views = _step_context(cache, runner, [(i, a, b) for i, (a, b) in enumerate(zip(first, second))])
    got2 = mix.forward(torch.cat([h[n:] for h, n in zip(hs, first)]).to(DEV).to(model.dtype), ctx, views[0]).float().cpu()
    at1 = at2 = 0
    for h, a, b in zip(hs, first, second):
        want = P.mixer(kind, h.double(), list(range(a + b)), W, "l0.mix.", mixer, 1e-6).float()
        got = torch.cat((got1[at1:at1 + a], got2[at2:at2 + b]))
        err = _rms_error(got, want)
        assert err < (1e-5 if dtype == "float32" else 3e-2), f"{kind} {mixer}: sequence of {a} + {b}: {err:.3e}"
        at1, at2 = at1 + a, at2 + b


# ---- a token made loud: what a wrong chunk, a lost page or a lost state would show --------------------------------
def _remember(w):
    """States that forget slowly, so that one token shows for hundreds of positions."""
    from tests.taluvik_helpers import spread
    spread(w)
    for name in w:
        if name.endswith("A_log"):
            w[name].sub_(4.0)


LOUD = [
    ("attention", _attn(4, 2, 64, 64, 50, 16, scale=0.2, softcap=20.0), (0, 15, 16, 49, 50, 99, 100, 249)),
    ("attention", _attn(2, 2, 32, 48, 48, 32, scale=0.3, softcap=6.0), (15, 16, 47, 48, 143, 144)),
    ("attention", _attn(2, 1, 20, 12, 128, 8, scale=0.3), (0, 63, 64, 127, 128)),
    ("delta", _delta(2, 1, 32, 24, 4), (0, 2, 3, 15, 16, 63, 64, 65, 127, 128, 250)),
    ("mamba1", _mamba(40, 6, 4, 3), (0, 1, 2, 15, 16, 63, 64, 65, 191, 192, 250)),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", range(len(LOUD)))
def test_a_loud_token_at_the_edges_of_chunks_pages_and_states(case, dtype):
    """One input row of the mixer is made twenty-five times as large as the others, so that what it leaves in the
    cache or the state dominates whatever reads it.  It sits at the sequence's first tokens, at both sides of a page's
    border, of a chunk of positions and of a chunk of the kernels, and far back; the outputs are computed as one prompt, as
    portions cut behind it and at the edge where it drops out of sight, decoded one by one across that edge, and in
    portions of two."""
    kind, mixer, places = LOUD[case]
    cfg = one_layer(kind, mixer, width=64)
    model, w = build(cfg, dtype, seed=9, edit=_remember)
    W = P.as_double(w)
    mix = model.blocks[0].mixer
    n = 300
    for loud in places:
        torch.manual_seed(loud)
        h = torch.randn(n, 64)
        h[loud] *= 25.0
        h = h.to(torch.bfloat16).float()
        want = P.mixer(kind, h.double(), list(range(n)), W, "l0.mix.", mixer, 1e-6).float()
        edge = (loud // mixer["mask"]["size"] + 1) * mixer["mask"]["size"] if kind == "attention" else loud + mixer["conv"]
        edge = min(edge, n - 2)
        cuts = {"whole": [n], "cut at the edge": [edge, 2, n], "cut right behind it": [loud + 1, 1, n],
                "decoded across the edge": [max(edge - 3, 1)] + [1] * 8 + [n], "portions of two": [max(edge - 5, 1)] + [2] * 5 + [n],
                "long portions": [loud + 40, 70, n]}
        for name, sizes in cuts.items():
            cache, runner = _session(model, blocks=40)
            got, at = [], 0
            for size in sizes:
                size = min(size, n - at)
                if size <= 0:
                    break
                ctx, views = _step_context(cache, runner, [("a", at, size)])
                got.append(mix.forward(h[at:at + size].to(DEV).to(model.dtype), ctx, views[0]).float().cpu())
                at += size
                cache.trim("a", at)
            got = torch.cat(got)
            assert at == n
            tol = 1e-5 if dtype == "float32" else 4e-2
            for lo, hi in ((0, n), (max(edge - 2, 0), min(edge + 4, n))):
                err = _rms_error(got[lo:hi], want[lo:hi])
                assert err < tol, f"{kind}, loud token at {loud}, {name}: positions {lo}..{hi}: {err:.3e}"
    # the loud token does show where it is seen (in the plain outputs that everything is held against)
    h = torch.randn(n, 64, generator=torch.Generator().manual_seed(1)).to(torch.bfloat16).double()
    loud = places[1]
    quiet = P.mixer(kind, h, list(range(n)), W, "l0.mix.", mixer, 1e-6)
    h2 = h.clone()
    h2[loud] *= 25.0
    shown = (P.mixer(kind, h2, list(range(n)), W, "l0.mix.", mixer, 1e-6) - quiet).abs().amax(1)
    edge = (loud // mixer["mask"]["size"] + 1) * mixer["mask"]["size"] if kind == "attention" else loud + 150
    assert float(shown[loud:edge].min()) > 1e-4 and (kind != "attention" or float(shown[edge:].max()) == 0.0)


def test_a_sink_outweighs_or_vanishes_per_head():
    """Heads whose sinks lie far above and far below their scores: the first give almost nothing, the others what they
    would without a sink."""
    mixer = _attn(2, 2, 16, 16, 0, 8, softcap=5.0)
    cfg = one_layer("attention", mixer, width=32)

    def edit(w):
        from tests.taluvik_helpers import spread
        spread(w)
        w["l0.mix.sink"].copy_(torch.tensor([12.0, -12.0]))
        w["l0.mix.o"].copy_(torch.eye(32))
    for dtype in DTYPES:
        model, w = build(cfg, dtype, edit=edit)
        h = torch.randn(20, 32).to(torch.bfloat16)
        cache, runner = _session(model)
        ctx, views = _step_context(cache, runner, [("a", 0, 20)])
        got = model.blocks[0].mixer.forward(h.to(DEV).to(model.dtype), ctx, views[0]).cpu()
        want = P.mixer("attention", h.double(), list(range(20)), P.as_double(w), "l0.mix.", mixer, 1e-6).float()
        assert _rms_error(got, want) < (1e-5 if dtype == "float32" else 3e-2)
        assert got[0, :16].norm() < 0.02 * got[0, 16:].norm()


# ---- whole models in the cuttings ----------------------------------------------------------------------
CUTS = {"whole": steps_whole, "decode": lambda r: steps_prefill_then_decode(r, tail=9), "portions": steps_portions}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cut", list(CUTS))
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_cuttings_against_plain(name, cut, dtype):
    cfg = CONFIGS[name]
    model, w = build(cfg, dtype, seed=11)
    reqs = {"x": tokens_for(cfg, 145, 1), "y": tokens_for(cfg, 1, 2), "z": tokens_for(cfg, 34, 3)}
    run_and_check(model, CUTS[cut](reqs), cfg, w, reqs, dtype, f"{name} {cut}", page_size=16 if name != "B" else 8, max_tokens=256)


def test_the_residual_stream_after_every_layer_run():
    """The float32 stream behind each layer run, layers that run again on shared weights among them."""
    cfg = CFG_A
    model, w = build(cfg, "float32", seed=3)
    toks = tokens_for(cfg, 70, 4)
    want = []
    P.forward(cfg, w, toks, want)
    from tensorline_amd.engine.batch import StepEntry
    cache, runner = _session(model)
    cache.add_request("a")
    cache.grow("a", 70)
    packed = runner.pack([StepEntry("a", toks, 0, [69])])
    ctx, views = runner.context(packed, runner._upload(packed.data))
    x, carry = model.embedding.forward(ctx.ids), None
    for e, view, after in zip(model.schedule, views, want):
        carry = model.blocks[e.layer].forward(x, carry, ctx, view)
        assert carry is None                       # nobody was named to take the branches: the block adds them itself
        assert _rms_error(x.double().cpu(), after) < 5e-6


@pytest.mark.parametrize("dtype", DTYPES)
def test_portions_down_to_two_tokens_and_one(dtype):
    cfg = CFG_A
    model, w = build(cfg, dtype, seed=4)
    reqs = {"x": tokens_for(cfg, 121, 5)}
    for sizes in ((2,), (1,), (2, 1, 3), (17, 2, 2, 1, 30), (65, 33, 2)):
        run_and_check(model, steps_portions(reqs, sizes=sizes), cfg, w, reqs, dtype, f"portions of {sizes}", max_tokens=128)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_mixed_batches_with_pages_and_slots_used_again(name, dtype):
    cfg = CONFIGS[name]
    model, w = build(cfg, dtype, seed=12)
    rng = random.Random(5)
    reqs = {f"r{i}": tokens_for(cfg, n, 20 + i) for i, n in enumerate([50, 3, 33, 1, 64, 17, 48, 2, 31])}
    # a pool that holds four live requests and no more: every page and slot is handed out several times
    run_and_check(model, mixed_steps(reqs, rng), cfg, w, reqs, dtype, f"{name} mixed", page_size=16, max_tokens=4 * 64, max_requests=4)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_request_alone_and_in_a_batch_of_unequal_requests(dtype):
    cfg = CFG_C
    model, w = build(cfg, dtype, seed=14)
    reqs = {"a": tokens_for(cfg, 90, 1), "b": tokens_for(cfg, 7, 2), "c": tokens_for(cfg, 41, 3)}
    alone = {r: run_steps(model, steps_portions({r: t}, sizes=(30, 1, 11)), max_tokens=256)[r] for r, t in reqs.items()}
    steps, at = [], {r: 0 for r in reqs}
    sizes = {"a": (30, 1, 11), "b": (2, 1), "c": (5, 25, 1)}
    k = 0
    while any(at[r] < len(reqs[r]) for r in reqs):
        entries, end = [], []
        for r, t in reqs.items():
            if at[r] < len(t):
                n = min(sizes[r][k % len(sizes[r])], len(t) - at[r])
                entries.append({"id": r, "tokens": t[at[r]:at[r] + n], "want": list(range(n))})
                at[r] += n
                if at[r] == len(t):
                    end.append(r)
        steps.append({"entries": entries, "end": end})
        k += 1
    together = run_steps(model, steps, max_tokens=256)
    tol = 1e-5 if dtype == "float32" else LIMIT[dtype]
    for r, t in reqs.items():
        for p in range(len(t)):
            assert rel_error(together[r][p], alone[r][p]) < tol, f"{r} at {p}: the batch changes a request's logits"


def test_the_first_tokens_and_a_slot_used_again():
    """A request of one token, then one of two, then one decoded from its first token on, all through one slot and
    the same few pages: nothing of an earlier request reaches the next."""
    cfg = CFG_A
    model, w = build(cfg, "float32", seed=6)
    reqs = {"p": tokens_for(cfg, 1, 1), "q": tokens_for(cfg, 2, 2), "r": tokens_for(cfg, 40, 3), "s": tokens_for(cfg, 5, 4)}
    steps = steps_whole({"p": reqs["p"], "q": reqs["q"]}) + steps_portions({"r": reqs["r"]}, sizes=(1,)) + steps_whole({"s": reqs["s"]})
    run_and_check(model, steps, cfg, w, reqs, "float32", "first tokens", max_tokens=64, max_requests=1)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_long_request_through_a_small_pool(dtype):
    """400 tokens in portions and then decoded, through chunks whose pages are given back as they pass, behind states that
    are carried all the way."""
    cfg = CFG_A
    model, w = build(cfg, dtype, seed=8)
    toks = tokens_for(cfg, 400, 7)
    steps, at = [], 0
    for n in [150, 130, 2, 60, 26] + [1] * 32:
        steps.append({"entries": [{"id": "a", "tokens": toks[at:at + n], "want": list(range(n))}], "end": ["a"] if at + n == len(toks) else []})
        at += n
    assert at == len(toks)
    run_and_check(model, steps, cfg, w, {"a": toks}, dtype, "400 tokens", max_tokens=448)


# ---- long decoding, graphs, the entry point ------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_eager_and_from_graphs(dtype):
    cfg = CFG_A
    model, w = build(cfg, dtype, seed=13)
    reqs = {"a": tokens_for(cfg, 150, 1), "b": tokens_for(cfg, 140, 2)}
    steps = [{"entries": [{"id": r, "tokens": t[:6], "want": list(range(6))} for r, t in reqs.items()], "end": []}]
    for i in range(6, 150):
        entries = [{"id": r, "tokens": [t[i]], "want": [0]} for r, t in reqs.items() if i < len(t)]
        steps.append({"entries": entries, "end": [r for r, t in reqs.items() if i == len(t) - 1]})
    run_and_check(model, copy.deepcopy(steps), cfg, w, reqs, dtype, "long decoding", max_tokens=512)
    from tensorline_amd.engine.replay import TraceSession
    plain_session, graph_session = TraceSession(model, 512), TraceSession(model, 512, graphs=True)
    plain_session.runner.fit_context = graph_session.runner.fit_context
    eager = run_steps(model, copy.deepcopy(steps), session=plain_session)
    replayed = run_steps(model, copy.deepcopy(steps), session=graph_session)
    assert graph_session.runner.graph_replays > 100
    for rid, toks in reqs.items():
        for p in range(len(toks)):
            assert rel_error(replayed[rid][p], eager[rid][p]) < 1e-6, f"{rid} at {p}: a graph's step differs from the eager one"


def _greedy(cfg, w, prompts, n):
    want = []
    for p in prompts:
        seq = list(p)
        for _ in range(n):
            seq.append(int(P.forward(cfg, w, seq)[-1].argmax()))
        want.append(seq[len(p):])
    return want


def _folder_weights(folder):
    from safetensors import safe_open
    w = {}
    with safe_open(folder + "/model.safetensors", "pt") as f:
        for k in f.keys():
            w[k] = f.get_tensor(k).float()
    return w


@pytest.mark.parametrize("name", ["A", "B"])
def test_greedy_generation_through_the_entry_point(name, tmp_path):
    """``LLM.generate`` with its scheduler, portions under a small token budget, more requests than slots at a
    time, and graphs: in 32-bit the greedy tokens are the plain implementation's."""
    from tensorline_amd import LLM, SamplingParams
    from tensorline_amd.weights.random_init import write_random_model
    cfg = CONFIGS[name]
    folder = write_random_model(typed(cfg), str(tmp_path / "model"), seed=21)
    w = _folder_weights(folder)
    prompts = [tokens_for(cfg, n, 40 + n) for n in (41, 3, 77, 18, 1, 30)]
    want = _greedy(cfg, w, prompts, 12)
    for options in (dict(graphs=False, max_batched_tokens=32, max_num_seqs=3), dict(graphs=True, max_batched_tokens=64, max_num_seqs=4)):
        llm = LLM(folder, dtype="float32", block_size=16 if name == "A" else 8, num_blocks=40 if name == "A" else 80,
                  max_model_len=128, graph_warmup_tokens=0, **options)
        outs = llm.generate(prompts, SamplingParams(max_tokens=12, temperature=0.0))
        assert [o.token_ids for o in outs] == want
        assert llm.cache.all_free()


def test_command_line_random_model_generate_and_trace_program(tmp_path):
    """The programs a user runs: ``tensorline random-model`` from a config.json, ``tensorline generate`` on the
    folder, and ``bin/trace_run`` fed steps on its standard input."""
    import json
    import os
    import subprocess
    import sys
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg = copy.deepcopy(CFG_B)
    (tmp_path / "cfg.json").write_text(json.dumps(cfg))
    tl = [sys.executable, os.path.join(root, "bin", "tensorline")]
    folder = str(tmp_path / "m")
    proc = subprocess.run(tl + ["random-model", "--config", str(tmp_path / "cfg.json"), "--out", folder, "--seed", "4"],
                          capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    w = _folder_weights(folder)
    prompts = [tokens_for(cfg, 19, 1), tokens_for(cfg, 4, 2)]
    want = _greedy(cfg, w, prompts, 6)
    base = tl + ["generate", "--model", folder, "--dtype", "float32", "--num-blocks", "32", "--block-size", "8",
                 "--max-tokens", "6", "--stop-token-id", "-1"]
    for p in prompts:
        base += ["--prompt-ids", " ".join(map(str, p))]
    proc = subprocess.run(base, capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    recs = [json.loads(l) for l in proc.stdout.splitlines() if l.startswith("{")]
    assert [r["token_ids"] for r in recs] == want
    toks = prompts[0]
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": toks[:7], "want": [6]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": toks[7:18], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": toks[18:], "want": [0]}], "end": ["a"]}]
    out = tmp_path / "out"
    proc = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", str(out),
                           "--max-tokens", "64"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                          capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    ref = P.forward(cfg, w, toks).numpy()
    assert not (out / "1.f32").exists()
    for step, place in ((0, 6), (2, 18)):
        got = np.fromfile(out / f"{step}.f32", dtype="<f4").reshape(1, -1)
        assert rel_error(got[0], ref[place]) < LIMIT["float32"]


# ---- seeded random configurations ----------------------------------------------------------------------------
@pytest.mark.parametrize("seed", range(16))
def test_random_configurations_in_mixed_batches(seed):
    """Sizes, head groupings, layer orders, layers that run again, chunks and constants drawn from the seed, a page size of 8,
    16 or 32, five requests cut at random over a pool that holds three: float32 for even seeds, bfloat16 for odd ones."""
    rng = random.Random(4000 + seed)
    cfg = random_config(rng)
    dtype = "float32" if seed % 2 == 0 else "bfloat16"
    model, w = build(cfg, dtype, seed=seed)
    reqs = {f"r{i}": tokens_for(cfg, n, 50 + i) for i, n in enumerate([rng.randint(1, 95) for _ in range(5)])}
    page = rng.choice([8, 16, 32])
    run_and_check(model, mixed_steps(reqs, rng, live=3), cfg, w, reqs, dtype, f"seed {seed}: {cfg}", page_size=page,
                  max_tokens=3 * 96, max_requests=3)
