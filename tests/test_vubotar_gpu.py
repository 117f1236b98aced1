"""Vubotar on the GPU against the plain implementation (tests/plain_vubotar.py): every mechanism alone, whole
prompts, token-by-token decoding, portions, mixed batches with pages and slots used again, tokens made to stand out
at the places where a cache, a state or a window can lose them, long decoding, and greedy generation through the
entry point."""
import copy
import random

import numpy as np
import pytest
import torch

from tests import plain_vubotar as P
from tests.helpers import steps_portions, steps_prefill_then_decode, steps_whole
from tests.samovik_helpers import rel_error, run_steps
from tests.test_samovik_gpu import mixed_steps
from tests.test_taluvik_gpu import _session, _Step, _step_context
from tests.tumitar_helpers import run_steps_with_routes
from tests.vubotar_helpers import (CFG_A, CFG_B, CFG_C, CONFIGS, _attn, _latent, _layer, _mlstm, _model, _moe, build, one_layer,
                                   random_config, routed_layers, spread, typed)

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = ["float32", "bfloat16"]
LIMIT = {"float32": 3e-5, "bfloat16": 5e-2}          # of the logits' own root mean square


def tokens_for(cfg, n, seed):
    rng = random.Random(seed)
    return [rng.randrange(cfg["vocab"]) for _ in range(n)]


def run_and_check(model, steps, cfg, w, reqs, dtype, what="", **kw):
    """Run the steps and hold every position against the plain implementation.  In float32 the plain run routes by
    itself.  In bfloat16 a router's close call may fall the other way and then changes every later position through
    the caches: there the plain run is told which experts the framework chose, and every such choice must be what
    the plain router chooses once its logits may move by a tenth of their spread."""
    if dtype == "float32":
        got, routes = run_steps(model, steps, **kw), {}
    else:
        got, routes = run_steps_with_routes(model, steps, **kw)
    layers = routed_layers(cfg)
    for rid, toks in reqs.items():
        forced = None
        if routes.get(rid):
            assert len(routes[rid]) == len(layers), f"{what}: the framework routed in {len(routes[rid])} layers, the model has {len(layers)}"
            forced = {layer: r.long() for layer, r in zip(layers, routes[rid])}
        seen = {}
        want = P.forward(cfg, w, toks, forced_experts=forced, router_logits=seen).numpy()
        for layer, taken in (forced or {}).items():
            z, correction = seen[layer], w[f"l{layer}.mlp.correction"].double()
            for t in range(len(toks)):
                slack = 0.1 * max(float(z[t].std()) if z.shape[1] > 1 else 1.0, 0.05)
                assert P.is_close_call(z[t], correction, taken[t], cfg["layers"][layer]["mlp"], slack), \
                    f"{what}: request {rid}, layer {layer}, position {t}: the experts {taken[t].tolist()} are not the router's choice"
        rows = got[rid]
        assert sorted(rows) == list(range(len(toks))), f"{what}: {rid} is missing positions"
        errs = {p: rel_error(rows[p], want[p]) for p in rows}
        first_bad = next((p for p in sorted(rows) if not errs[p] <= LIMIT[dtype]), None)
        assert first_bad is None, (f"{what} {dtype}: request {rid}: first wrong position {first_bad} of {len(toks)}, "
                                   f"worst error {max(errs.values()):.3e}")


def _rms_error(got, want):
    return ((got - want).pow(2).mean().sqrt() / want.pow(2).mean().sqrt().clamp(min=1e-30)).item()


# ---- every mechanism alone -------------------------------------------------------------------------
@pytest.mark.parametrize("H", [4, 96, 130, 1000, 4096, 5121])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_branches_join_the_stream_and_two_norms_read_it(H, dtype):
    """Plain branches, a product in shares, experts' rows with weights; with and without factors; one norm, two and none."""
    from tensorline_amd.ops import kernels
    torch.manual_seed(H)
    T, top = 600 if H == 4096 else 7, 3
    x, y1, y2, w1, w2, s1, s2 = torch.randn(T, H), torch.randn(T, H), torch.randn(T, H), *(torch.randn(H) for _ in range(4))
    rows, weights = torch.randn(T * top, H), torch.rand(T, top)
    g, d = lambda t: t.to(DEV), lambda t: t.double()
    mixed = (d(rows).view(T, top, H) * d(weights)[:, :, None]).sum(1)
    cases = [
        (None, d(x)), (g(y1), d(x) + d(y1)), (kernels.ShareSum(g(torch.stack((y1, y2, y1)))), d(x) + 2 * d(y1) + d(y2)),
        (kernels.JoinedBranches(g(y1), g(s1)), d(x) + d(s1) * d(y1)),
        (kernels.JoinedBranches(g(y1), g(s1), g(y2), g(s2)), d(x) + d(s1) * d(y1) + d(s2) * d(y2)),
        (kernels.JoinedBranches(kernels.ShareSum(g(torch.stack((y1, y2)))), None, kernels.ExpertRows(g(rows), g(weights)), g(s2)),
         d(x) + d(y1) + d(y2) + d(s2) * mixed),
    ]
    tol = dict(atol=2e-5, rtol=2e-5) if dtype == torch.float32 else dict(atol=3e-2, rtol=1e-2)
    for branches, total in cases:
        for second in (g(w2), None):
            got_x = g(x).clone()
            a, b = kernels.join_norms(got_x, branches, g(w1), second, 1e-5, dtype)
            torch.testing.assert_close(got_x.double().cpu(), total, atol=2e-5, rtol=1e-5)
            torch.testing.assert_close(a.double().cpu(), P.rms_norm(total, d(w1), 1e-5), **tol)
            assert (b is None) == (second is None)
            if b is not None:
                torch.testing.assert_close(b.double().cpu(), P.rms_norm(total, d(w2), 1e-5), **tol)
        some = torch.tensor([T - 1, 0, 2], dtype=torch.int32, device=DEV)
        got_x = g(x).clone()
        a, _ = kernels.join_norms(got_x, branches, g(w1), None, 1e-5, dtype, rows=some)
        assert torch.equal(got_x.cpu(), x)
        torch.testing.assert_close(a.double().cpu(), P.rms_norm(total[some.cpu().long()], d(w1), 1e-5), **tol)
        if branches is not None:
            got_x = g(x).clone()
            assert kernels.join_norms(got_x, branches, None, None, 0.0, None) == (None, None)
            torch.testing.assert_close(got_x.double().cpu(), total, atol=2e-5, rtol=1e-5)


@pytest.mark.parametrize("n", [1, 7, 64, 300])
def test_norm_of_a_block_of_columns_and_capped_logits(n):
    from tensorline_amd.ops import kernels
    torch.manual_seed(n)
    wide, w = torch.randn(5, n + 9), torch.randn(n)
    for dtype in (torch.float32, torch.bfloat16):
        got = kernels.norm_rows(wide.to(DEV)[:, 4:4 + n], w.to(DEV), 1e-6, dtype).double().cpu()
        tol = 1e-5 if dtype == torch.float32 else 2e-2
        torch.testing.assert_close(got, P.rms_norm(wide[:, 4:4 + n].double(), w.double(), 1e-6), atol=tol, rtol=tol)
    z = torch.randn(3, n) * 40
    for scale, cap in ((0.3, 5.0), (1.0, 30.0), (2.5, 0.0)):
        got = kernels.scale_cap(z.to(DEV).clone(), scale, cap).double().cpu()
        torch.testing.assert_close(got, P.bend(z.double() * scale, cap), atol=1e-5, rtol=1e-5)


MLSTM_LENS = [[1, 1, 1], [33, 1, 64], [2, 150, 65, 700], [32, 31]]


@pytest.mark.parametrize("case", [(2, 24, 40), (1, 7, 9), (3, 128, 72), (1, 256, 16), (2, 64, 144), (1, 130, 200), (5, 16, 16), (2, 1, 1)])
@pytest.mark.parametrize("lens", range(len(MLSTM_LENS)))
@pytest.mark.parametrize("chunked", [False, True])
def test_matrix_memory_token_by_token_and_in_chunks(case, lens, chunked):
    """Sequences of 1 to 700 tokens from states of their own (a running maximum above and below zero), gates from wide open to
    closed, against the plain walk continued from the same state; other slots stay as they were."""
    from tensorline_amd.ops import kernels
    H, dk, dv = case
    lens = MLSTM_LENS[lens]
    step = _Step(lens, chunked)
    if chunked and step.chunks is None:
        pytest.skip("nothing long enough for chunks")
    torch.manual_seed(sum(case) + len(lens))
    T, cap = sum(lens), 6.0
    q, k, v = torch.randn(T, H * dk) * 0.5, torch.randn(T, H * dk), torch.randn(T, H * dv)
    gi, gf = torch.randn(T, H) * 4, torch.randn(T, H) * 4 + 2
    gf[T // 2:T // 2 + 3] = -30.0                          # gates that close inside a sequence
    bi, bf = torch.randn(H), torch.randn(H)
    size, nb, slots = kernels.matrix_lstm_state(H, dk, dv), -(-dv // 16), len(lens) + 2
    state = torch.randn(slots, size + 3) * 0.3
    S0 = state[:, :H * dv * dk].view(slots, H, dv, dk)
    n0 = torch.randn(slots, H, dk)
    m0 = torch.randn(slots, H) * 2
    state[:, H * dv * dk:H * dv * dk + H * nb * dk] = n0.repeat_interleave(nb, 1).reshape(slots, -1)
    state[:, H * (dv * dk + nb * dk):size] = m0.repeat_interleave(nb, 1)
    proj = torch.cat([q, k, v, gi, gf], 1).to(DEV)
    cols = np.cumsum([0, H * dk, H * dk, H * dv, H, H])
    part = [proj[:, a:b] for a, b in zip(cols, cols[1:])]
    arena = state.to(DEV).clone()
    got = kernels.matrix_lstm(*part, bi.to(DEV), bf.to(DEV), cap, step, arena, H, dk, dv, q_scale=0.7, chunks=step.chunks).double().cpu()
    after = arena.cpu()
    at = 0
    for s, n in enumerate(lens):
        slot = int(step.state_slots[s])
        for h in range(H):
            i = P.bend(gi[at:at + n, h].double() + bi[h].double(), cap)
            f = [P.log_sigmoid(float(z)) for z in P.bend(gf[at:at + n, h].double() + bf[h].double(), cap)]
            S, nn, m = S0[slot, h].double().T.clone(), n0[slot, h].double().clone(), float(m0[slot, h])
            S_abs, n_abs = S.abs(), nn.abs()               # the same sums with every term's size
            want, room = torch.zeros(n, dv, dtype=torch.float64), torch.zeros(n, dtype=torch.float64)
            for t in range(n):
                kt, vt, qt = (x[at + t, h * w:(h + 1) * w].double() for x, w in ((k, dk), (v, dv), (q, dk)))
                new = max(f[t] + m, float(i[t]))
                keep, add = np.exp(f[t] + m - new), np.exp(float(i[t]) - new)
                S, nn, m = keep * S + add * torch.outer(kt, vt), keep * nn + add * kt, new
                S_abs, n_abs = keep * S_abs + add * torch.outer(kt, vt).abs(), keep * n_abs + add * kt.abs()
                den = max(abs(0.7 * float(nn @ qt)), np.exp(-m)) + 1e-6
                want[t] = (0.7 * qt) @ S / den
                # n . q may pass through zero, where the output is large and its digits few: what the sums' terms allow
                room[t] = 0.7 * (float((qt.abs() @ S_abs).max()) + float(want[t].abs().max()) * float(qt.abs() @ n_abs)) / den
            g = got[at:at + n, h * dv:(h + 1) * dv]
            err = ((g - want).abs().amax(1) / room.clamp(min=1e-3)).max()
            assert err < 5e-6, f"sequence {s} of {n}, head {h}: {err:.2e}"
            # the state, as a true sum: the running maximum is a scale that rounding may shift
            got_m = after[slot, H * (dv * dk + nb * dk) + h * nb:H * (dv * dk + nb * dk) + (h + 1) * nb].double()
            assert (got_m - m).abs().max() < 1e-5 and (got_m == got_m[0]).all()
            got_S = after[slot, :H * dv * dk].view(H, dv, dk)[h].double().T
            assert (got_S - S).abs().max() < 2e-5 * max(1.0, float(S.abs().max()))
            got_n = after[slot, H * dv * dk:H * dv * dk + H * nb * dk].view(H, nb, dk)[h].double()
            assert (got_n - nn).abs().max() < 2e-5 * max(1.0, float(nn.abs().max())) and (got_n == got_n[0]).all()
        at += n
    used = {int(x) for x in step.state_slots}
    for slot in range(slots):
        if slot not in used:
            assert torch.equal(after[slot], state[slot])
    assert torch.equal(after[:, size:], state[:, size:])


def test_a_forget_gate_that_closes_costs_no_digits_between_its_neighbours():
    """Log decays of dozens inside one chunk, then tokens that barely forget: what they give to each other is exact."""
    from tensorline_amd.ops import kernels
    torch.manual_seed(0)
    T, dk, dv, cap = 64, 8, 16, 60.0
    q, k, v = torch.randn(T, dk), torch.randn(T, dk), torch.randn(T, dv)
    gi, gf = torch.randn(T, 1) * 0.1, torch.full((T, 1), 4.0)
    gf[:40:2] = -58.0
    step = _Step([T], True)
    arena = torch.zeros(1, kernels.matrix_lstm_state(1, dk, dv), device=DEV)
    got = kernels.matrix_lstm(*(t.to(DEV) for t in (q, k, v, gi, gf)), None, None, cap, step, arena, 1, dk, dv, chunks=step.chunks).double().cpu()
    i, f = P.bend(gi.double(), cap)[:, 0], torch.tensor([P.log_sigmoid(float(z)) for z in P.bend(gf.double(), cap)])
    want = P.mlstm_walk(q.double(), k.double(), v.double(), i, f)
    assert ((got - want).abs().amax(1) / want.abs().amax(1).clamp(min=0.05)).max() < 1e-4


@pytest.mark.parametrize("case", [(4, 2, 24, 40), (3, 1, 10, 7), (2, 2, 128, 128), (5, 5, 250, 200)])
@pytest.mark.parametrize("T", [5, 100])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_values_mixed_on_their_way_into_the_cache(case, T, dtype):
    from tensorline_amd.ops import kernels
    H, G, d, dv = case
    D, page, pages = -(-max(d, dv) // 16) * 16, 8, 16
    torch.manual_seed(sum(case))
    proj, first = torch.randn(T, (H + G) * d + G * dv + 3), torch.randn(T, 5 + G * dv)
    slots = torch.randperm(pages * page)[:T].to(torch.int32)
    wq, wk = torch.randn(d) + 1, torch.randn(d) + 1
    kc = torch.full((pages, page, G, D), 7.0).to(dtype).to(DEV)
    vc = torch.full((pages, G, D, page), 7.0).to(dtype).to(DEV)
    kernels.head_norm_rotate_store(proj.to(DEV), slots.to(DEV), wq.to(DEV), wk.to(DEV), 1e-5, None, 1.0, kc, vc, slots.to(DEV), H, G, d, dv,
                                   False, dtype, first_values=first.to(DEV)[:, 5:], mix=0.3)
    want = 0.7 * proj[:, (H + G) * d:(H + G) * d + G * dv].double() + 0.3 * first[:, 5:].double()
    got = vc.double().cpu().permute(0, 3, 1, 2).reshape(-1, G, D)[slots.long()]
    tol = 1e-5 if dtype == torch.float32 else 3e-2
    torch.testing.assert_close(got[:, :, :dv], want.view(T, G, dv), atol=tol, rtol=tol)
    assert not got[:, :, dv:].any()
    keys = kc.double().cpu().view(-1, G, D)[slots.long()][:, :, :d]
    torch.testing.assert_close(keys, P.rms_norm(proj[:, H * d:(H + G) * d].double().view(T, G, d), wk.double(), 1e-5), atol=max(tol, 1e-4), rtol=tol)


@pytest.mark.parametrize("experts,top", [(15, 5), (8, 3), (6, 6), (128, 9), (200, 32), (4, 1), (64, 5), (1, 1), (1000, 4)])
def test_router_chooses_by_corrected_scores(experts, top):
    from tensorline_amd.ops import kernels
    torch.manual_seed(experts)
    z = (torch.randn(40, experts + 3) * 2).float()
    correction = torch.randn(experts) * 0.5 - 0.6          # sums of either sign
    z[1, :experts] = 0.25
    correction[experts // 2:] = correction[experts // 2]   # ties: the lower index wins
    ids, wts = kernels.moe_route(z.to(DEV), top, "sigmoid_grouped", experts=experts, correction=correction.to(DEV))
    for t in range(z.shape[0]):
        # in float32, as the choice is: ties stay ties
        s = torch.sigmoid(z[t, :experts])
        chosen, weights = P.route(z[t, :experts].float(), correction, top)
        if ids[t].tolist() != chosen:                       # the sigmoid's last digit may part two that are equal here
            assert torch.allclose((s + correction)[ids[t].cpu().long()].sort().values, (s + correction)[chosen].sort().values, atol=1e-6), f"row {t}"
            continue
        assert torch.allclose(wts[t].cpu().double(), torch.tensor(weights, dtype=torch.float64), atol=1e-6)
    assert torch.allclose(wts.sum(1).cpu(), torch.ones(z.shape[0]), atol=1e-5)


def test_correction_chooses_groups_too():
    """The group whose two best corrected scores sum highest is kept, also where the sums are negative."""
    from tensorline_amd.ops import kernels
    z = torch.tensor([[4.0, -9.0, -9.0, 1.5, 1.4, 1.3]])
    for correction, want in ((torch.zeros(6), [3, 4]), (torch.tensor([0.0, 0.0, 0.0, -1.0, -1.0, -1.0]), [0, 1]),
                             (torch.tensor([-3.0, -3.0, -2.0, -2.0, -3.0, -2.5]), [3, 5])):
        ids, wts = kernels.moe_route(z.to(DEV), 2, "sigmoid_grouped", groups=2, keep=1, correction=correction.to(DEV))
        assert ids.tolist() == [want]
        s = torch.sigmoid(z[0].double())[want]
        assert torch.allclose(wts[0].cpu().double(), s / s.sum(), atol=1e-6)


MIXERS = [
    ("attention", _attn(4, 2, 24, 40, 21, 3)),
    ("attention", _attn(1, 1, 10, 10, 3, bias_max=2, rows=2, softcap=None)),           # small and odd, nothing kept, a table of two rows
    ("attention", _attn(6, 1, 64, 64, 40, 20, bias_max=30, rows=9)),                    # matrix-core attention, more kept than a page
    ("attention", _attn(2, 2, 128, 96, 500, 4, bias_max=128, rows=32, scale=0.05)),      # a window wider than the sequence
    ("attention", _attn(18, 2, 32, 16, 100, 1, bias_max=64, rows=6, softcap=2.0)),       # nine query heads a group
    ("attention", _attn(4, 4, 48, 48, 16, 16, bias_max=17, rows=32)),                   # a table that is nearly linear
    ("attention", _attn(4, 1, 64, 64, 0, bias_max=2000, rows=32)),                      # no window, a reach beyond the sequence
    ("attention", _attn(28, 2, 64, 32, 0, bias_max=2900, rows=20)),                     # a table wider than LDS holds
    ("latent_attention", _latent(3, 16, 8, 24, 20, 40)),
    ("latent_attention", _latent(1, 6, 2, 9, 1, 11)),
    ("latent_attention", _latent(4, 32, 16, 32, 24, 136, base=10000.0)),                 # a cached row of 256
    ("latent_attention", _latent(2, 24, 32, 16, 40, 96, base=50.0)),                     # a cached row of 128
    ("latent_attention", _latent(2, 16, 8, 8, 9, 300)),                                  # wider than the matrix-core kernels take
    ("mlstm", _mlstm(2, 24, 40)), ("mlstm", _mlstm(1, 7, 9, 2.0)), ("mlstm", _mlstm(3, 128, 72)), ("mlstm", _mlstm(4, 64, 144)),
    ("mlstm", _mlstm(1, 200, 24, 15.0)),
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
        assert err < (2e-5 if dtype == "float32" else 3e-2), f"{kind} {mixer}: sequence of {a} + {b}: {err:.3e}"
        at1, at2 = at1 + a, at2 + b


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mlp", [_moe(6, 2, 40), _moe(3, 3, 20), _moe(1, 1, 100), _moe(40, 5, 16)])
def test_feed_forward_alone(mlp, dtype):
    """Few rows and many (the grouped product's tiles of 16 and of 64 rows), added up and left as rows."""
    from tensorline_amd.ops import kernels
    cfg = one_layer("mlstm", _mlstm(1, 8, 8), mlp, width=88)
    model, w = build(cfg, dtype, seed=3)
    W = P.as_double(w)
    ff = model.blocks[0].feed_forward
    for rows in (1, 5, 300):
        torch.manual_seed(rows)
        h = (torch.randn(rows, 88) * 2).to(torch.bfloat16).float()
        want = P.ff_experts(h.double(), W, "l0.mlp.", mlp).float()
        dev_h = h.to(DEV).to(model.dtype)
        got = ff.forward(dev_h, None).float().cpu()
        kept = ff.forward(dev_h, None, keep_rows=True)
        assert isinstance(kept, kernels.ExpertRows)
        summed = (kept.rows.view(rows, -1, 88) * kept.weights[:, :, None]).sum(1).cpu()
        for y in (got, summed):
            err = (y - want).abs().max().item() / want.abs().max().item()
            assert err < (1e-5 if dtype == "float32" else 3e-2), f"{rows} rows: {err:.3e}"


# ---- a token made loud: what a wrong window, bias, kept token, lost page or lost state would show ------------------
def _remember(w):
    """States that forget slowly, so that one token shows for hundreds of positions; keys and queries that let one key stand out
    from hundreds."""
    spread(w)
    for name in w:
        if name.endswith("f.b"):
            w[name].add_(4.0)


LOUD = [
    ("attention", _attn(4, 2, 64, 64, 37, 5, bias_max=30, rows=8, scale=0.4, softcap=30.0), (0, 4, 5, 15, 16, 31, 230)),
    ("attention", _attn(2, 1, 32, 32, 48, 18, bias_max=200, rows=32, scale=0.5, softcap=40.0), (0, 16, 17, 18, 47, 48, 100)),
    ("attention", _attn(2, 2, 20, 12, 128, 1, bias_max=12, rows=9, scale=0.5), (0, 1, 63, 64, 127, 128)),
    ("latent_attention", _latent(4, 32, 16, 32, 24, 48, scale=0.2), (0, 15, 16, 31, 230)),
    ("latent_attention", _latent(2, 16, 8, 16, 24, 150, scale=0.3), (0, 63, 64, 200)),
    ("mlstm", _mlstm(2, 32, 24, 9.0), (0, 1, 15, 16, 31, 32, 63, 64, 65, 127, 128, 250)),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", range(len(LOUD)))
def test_a_loud_token_at_the_edges_of_windows_pages_and_states(case, dtype):
    """One input row of the mixer is made twenty-five times as large as the others, so that what it leaves in the
    cache or the state dominates whatever reads it.  It sits at the sequence's first tokens, among the kept ones and right
    behind them, at both sides of a page's border, of a window's edge and of a chunk of the kernels, and far back; the outputs are
    computed as one prompt, as portions cut behind it and at the edge where it drops out of sight, decoded one by one across
    that edge, and in portions of two, with pages given back as the layer allows."""
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
        edge = loud + 3
        if kind == "attention" and loud >= mixer["mask"].get("keep_first", 0):
            edge = loud + mixer["mask"]["size"]
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
            tol = 2e-5 if dtype == "float32" else 4e-2
            for lo, hi in ((0, n), (max(edge - 2, 0), min(edge + 4, n))):
                err = _rms_error(got[lo:hi], want[lo:hi])
                assert err < tol, f"{kind}, loud token at {loud}, {name}: positions {lo}..{hi}: {err:.3e}"
    # the loud token does show where it is seen, and only there (in the plain outputs that everything is held against)
    h = torch.randn(n, 64, generator=torch.Generator().manual_seed(1)).to(torch.bfloat16).double()
    loud = places[-2]
    quiet = P.mixer(kind, h, list(range(n)), W, "l0.mix.", mixer, 1e-6)
    h2 = h.clone()
    h2[loud] *= 25.0
    shown = (P.mixer(kind, h2, list(range(n)), W, "l0.mix.", mixer, 1e-6) - quiet).abs().amax(1)
    edge = loud + mixer["mask"]["size"] if kind == "attention" else min(loud + 100, n)
    assert float(shown[loud:min(edge, n)].min()) > 1e-5 and (kind != "attention" or edge >= n or float(shown[edge:].max()) == 0.0)


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


@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_the_residual_stream_after_every_layer(name):
    """The float32 stream behind each layer, whether the block hands its branches on or adds them itself."""
    cfg = CONFIGS[name]
    model, w = build(cfg, "float32", seed=3)
    toks = tokens_for(cfg, 70, 4)
    _, want = P.forward(cfg, w, toks, want_layers=True)
    from tensorline_amd.engine.batch import StepEntry
    from tensorline_amd.ops import kernels
    from tensorline_amd.parts.spec import Intake
    cache, runner = _session(model)
    cache.add_request("a")
    cache.grow("a", 70)
    packed = runner.pack([StepEntry("a", toks, 0, [69])])
    for after in (None, Intake(joined_branches=True)):
        ctx, views = runner.context(packed, runner._upload(packed.data))
        x, carry = model.embedding.forward(ctx.ids), None
        for e, view, stream in zip(model.schedule, views, want):
            if view.state is not None:
                view.state.zero_()
            carry = model.blocks[e.layer].forward(x, carry, ctx, view, after=after)
            assert isinstance(carry, kernels.JoinedBranches) == (after is not None)
            there = x.clone()
            if carry is not None:
                kernels.join_norms(there, carry, None, None, 0.0, None)
            assert _rms_error(there.double().cpu(), stream) < 1e-5


@pytest.mark.parametrize("dtype", DTYPES)
def test_portions_down_to_two_tokens_and_one(dtype):
    cfg = CFG_A
    model, w = build(cfg, dtype, seed=4)
    reqs = {"x": tokens_for(cfg, 121, 5)}
    for sizes in ((2,), (1,), (2, 1, 3), (17, 2, 2, 1, 30), (70, 2, 49)):
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
def test_long_portions_beside_decoded_tokens(dtype):
    """Portions taken in chunks, short ones that are walked and single tokens in one batch, through layers that share values."""
    cfg = CFG_A
    model, w = build(cfg, dtype, seed=15)
    reqs = {"a": tokens_for(cfg, 260, 1), "b": tokens_for(cfg, 90, 2), "c": tokens_for(cfg, 12, 3)}
    sizes = {"a": [100, 33, 65, 2, 60], "b": [1, 1, 80, 7, 1], "c": [5, 1, 1, 4, 1]}
    steps, at = [], {r: 0 for r in reqs}
    for i in range(5):
        entries = []
        for r in reqs:
            n = sizes[r][i]
            entries.append({"id": r, "tokens": reqs[r][at[r]:at[r] + n], "want": list(range(n))})
            at[r] += n
        steps.append({"entries": entries, "end": [r for r in reqs if at[r] == len(reqs[r])]})
    assert all(at[r] == len(reqs[r]) for r in reqs)
    run_and_check(model, steps, cfg, w, reqs, dtype, "long portions", max_tokens=512)


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
    tol = 2e-5 if dtype == "float32" else LIMIT[dtype]
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
    """400 tokens in portions and then decoded, with pages given back as windows pass; the kept first tokens and the latent
    rows are read hundreds of positions later."""
    cfg = CFG_C
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
    folder (whose config.json leaves the distance tables' rows to the tensors), and ``bin/trace_run`` fed steps on its standard
    input."""
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
    raw = json.loads((tmp_path / "m" / "config.json").read_text())
    for layer in raw["layers"]:
        layer["mixer"].pop("bias_rows", None)
    (tmp_path / "m" / "config.json").write_text(json.dumps(raw))
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
    """Sizes, head groupings, layer orders, windows, kept tokens, reaches and constants drawn from the seed, a page size
    of 8, 16 or 32, five requests cut at random over a pool that holds three: float32 for even seeds, bfloat16 for
    odd ones."""
    rng = random.Random(4000 + seed)
    cfg = random_config(rng)
    dtype = "float32" if seed % 2 == 0 else "bfloat16"
    model, w = build(cfg, dtype, seed=seed)
    reqs = {f"r{i}": tokens_for(cfg, n, 50 + i) for i, n in enumerate([rng.randint(1, 90) for _ in range(5)])}
    page = rng.choice([8, 16, 32])
    run_and_check(model, mixed_steps(reqs, rng, live=3), cfg, w, reqs, dtype, f"seed {seed}: {cfg}", page_size=page,
                  max_tokens=3 * 96, max_requests=3)
