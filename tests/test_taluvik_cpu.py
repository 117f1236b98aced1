"""Taluvik without a GPU: the configuration reader and what it refuses, the spec (mixer kinds, run order, cache and state
needs, tensor names), the tables of chunks a step brings, and pins of the plain implementation (tests/plain_taluvik.py)
against closed forms."""
import copy
import math

import pytest
import torch

from tensorline_amd.config.model_config import ConfigError
from tensorline_amd.config.registry import get_architecture, known_architectures
from tensorline_amd.engine.batch import StepFacts
from tensorline_amd.models.decoder import DecoderModel
from tensorline_amd.ops import kernels
from tensorline_amd.parts.rotary import band_frequencies, rotation_frequencies, yarn_frequencies
from tensorline_amd.weights.random_init import random_tensor
from tests import plain_taluvik as P
from tests.taluvik_helpers import BANDS, CFG_A, CFG_B, CFG_C, _attn, _delta, _layer, _mamba, one_layer, typed


def _model(cfg):
    return DecoderModel(get_architecture("Taluvik").build_spec(typed(cfg)), torch.float32, "cpu")


def _weights(cfg, seed=0):
    return {n: random_tensor(n, d, seed, "cpu").to(torch.float64) for n, d in _model(cfg).tensor_decls().items()}


def test_registered_and_round_trips():
    assert "Taluvik" in known_architectures()
    for cfg in (CFG_A, CFG_B, CFG_C):
        t = typed(cfg)
        assert typed(t.to_dict()) == t


@pytest.mark.parametrize("edit, text", [
    (lambda c: c["layers"][0].update(type="mamba3"), "unknown"),
    (lambda c: c["layers"][0]["mixer"].pop("conv"), "conv must be"),
    (lambda c: c["layers"][1]["mixer"].update(state=0), "state must be"),
    (lambda c: c["layers"][0]["mixer"].update(heads=3), "not a multiple"),
    (lambda c: c["layers"][2]["mixer"].pop("scale"), "scale must be"),
    (lambda c: c["layers"][2]["mixer"].update(softcap=-1.0), "softcap must be"),
    (lambda c: c["layers"][2]["mixer"]["rot"].update(dims=7), "even"),
    (lambda c: c["layers"][2]["mixer"]["rot"]["scaling"].pop("high"), "high must be"),
    (lambda c: c["layers"][2]["mixer"]["mask"].update(size=0), "size must be"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "unknown"),
    (lambda c: c["layers"][4].update(weights_of=4), "another layer"),
    (lambda c: c["layers"][4].update(weights_of=9), "another layer"),
    (lambda c: c["layers"][4].update(weights_of=0), "type differs"),
    (lambda c: c["layers"][5].update(mlp=None), "mlp differs"),
    (lambda c: (c["layers"][0].update(weights_of=5)), "leads back"),
    (lambda c: c.pop("norm"), "norm.eps"),
])
def test_reader_refuses(edit, text):
    cfg = copy.deepcopy(CFG_A)
    edit(cfg)
    with pytest.raises(ConfigError, match=text):
        typed(cfg)


def test_spec_kinds_run_order_needs_and_names():
    m = _model(CFG_A)
    assert [type(b.mixer).__name__ for b in m.blocks] == ["GatedDeltaRule", "SelectiveScan", "MaskedAttention", "GatedDeltaRule"]
    assert [e.layer for e in m.schedule] == [0, 1, 2, 3, 1, 0, 2]           # a run of its own for every layer of the list
    assert all(e.cache_from is None for e in m.schedule)
    states, caches = m.state_needs(), m.cache_needs()
    assert len(states) == len(caches) == 7
    assert states[0].shape == (4 * 40 * 24 + 3 * (2 * 2 * 24 + 4 * 40),) == states[5].shape
    assert states[1].shape == (88 * 12 + 3 * 88,) == states[4].shape and states[2] is None
    assert [c.chunk if c else None for c in caches] == [None, None, 19, None, None, None, 19]
    assert caches[2].planes[0].shape == (2, 48)                              # ceil16(max(dim, vdim))
    names = set(m.tensor_decls())
    assert {"embed", "head", "final.norm", "final.norm.b", "l0.norm1", "l0.norm1.b", "l0.mix.q.conv", "l0.mix.b", "l0.mix.a",
            "l1.mix.conv.b", "l1.mix.dt.b", "l1.mix.D", "l2.mix.sink", "l3.mix.o"} <= names
    assert not {n for n in names if n.startswith(("l4.", "l5.", "l6.")) or "norm2" in n or n.startswith("l3.mlp")}
    decls = m.tensor_decls()
    assert decls["l1.mix.x"].shape == (8 + 24, 88) and decls["l1.mix.A_log"].shape == (88, 12) and decls["l2.mix.sink"].shape == (4,)
    assert decls["l0.mix.norm"].shape == (40,) and decls["head"].shape == (320, 96)


def test_chunks_of_a_step():
    facts = StepFacts(max_context=300, max_query_len=130, num_seqs=4, q_lens=[130, 1, 64], starts=[0, 40, 7])
    v = kernels.chunk_vectors(facts)
    # the sequence of one token and the padding sequence are walked
    assert v["chunks.seq"] == [0, 0, 0, 2] and v["chunks.row"] == [0, 64, 128, 131]
    assert v["chunks.first"] == [0, 3, 3, 4, 4]
    assert kernels.chunk_vectors(StepFacts(max_query_len=1, decode_only=True, num_seqs=2, q_lens=[1, 1], starts=[5, 6])) == {}
    assert kernels.chunk_vectors(StepFacts(max_query_len=32, num_seqs=1, q_lens=[32], starts=[0])) == {}
    # every part that takes chunks asks for the same tables
    assert set(_model(CFG_A).step_vectors(facts)) == {"attention.single_seqs", "chunks.seq", "chunks.row", "chunks.first"}


# ---- pins of the plain implementation ---------------------------------------------------------------------
def test_band_frequencies_of_the_framework_are_the_plain_ones():
    for dims, base, scaling in ((8, 500.0, BANDS), (64, 50000.0, {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 512}),
                                (20, 50.0, None), (2, 10.0, BANDS)):
        want = torch.tensor(P.frequencies(dims, base, scaling), dtype=torch.float64)
        assert torch.allclose(band_frequencies(dims, base, scaling).double(), want, rtol=1e-6)
        f, mag = rotation_frequencies(dims, base, scaling)
        assert torch.allclose(f.double(), want, rtol=1e-6) and mag == 1.0
    yarn = {"factor": 4.0, "original": 64, "fast": 16.0, "slow": 2.0}
    assert torch.equal(rotation_frequencies(8, 500.0, yarn)[0], yarn_frequencies(8, 500.0, yarn)[0])
    # a wave of many turns keeps its frequency, one of less than `low` turns is stretched by the factor
    f = P.frequencies(4, 1e6, {"factor": 5.0, "low": 1.0, "high": 2.0, "original": 100})
    assert f[0] == 1.0 and abs(f[1] - 1e-3 / 5.0) < 1e-15


def test_layer_norm_and_unit_rows():
    x = torch.tensor([[1.0, 3.0, 5.0, 7.0]], dtype=torch.float64)
    one, zero = torch.ones(4, dtype=torch.float64), torch.zeros(4, dtype=torch.float64)
    assert torch.allclose(P.layer_norm(x, one, zero, 0.0), (x - 4.0) / math.sqrt(5.0))
    assert torch.allclose(P.layer_norm(x, 2 * one, one, 0.0), 2 * (x - 4.0) / math.sqrt(5.0) + 1.0)
    assert torch.allclose(P.unit_rows(torch.tensor([[3.0, 4.0]], dtype=torch.float64)), torch.tensor([[0.6, 0.8]], dtype=torch.float64), atol=1e-7)
    assert float(P.unit_rows(torch.zeros(1, 2, dtype=torch.float64)).abs().max()) == 0.0


def test_rotation_turns_halves_and_leaves_the_rest():
    x = torch.arange(1.0, 7.0, dtype=torch.float64).view(1, 1, 6)
    got = P.turn_halves(x.repeat(2, 1, 1), [0, 3], [0.5, 2.0])
    assert torch.equal(got[0], x[0])
    a, b = 1.5, 6.0
    want = torch.tensor([1 * math.cos(a) - 3 * math.sin(a), 2 * math.cos(b) - 4 * math.sin(b), 3 * math.cos(a) + 1 * math.sin(a),
                         4 * math.cos(b) + 2 * math.sin(b), 5.0, 6.0], dtype=torch.float64)
    assert torch.allclose(got[1, 0], want)


def test_convolution_reads_zeros_ahead_of_the_sequence():
    x = torch.tensor([[1.0], [10.0], [100.0]], dtype=torch.float64)
    taps = torch.tensor([[2.0, 3.0, 5.0]], dtype=torch.float64)
    assert P.causal_conv(x, taps)[:, 0].tolist() == [5.0, 53.0, 532.0]
    assert P.causal_conv(x, taps, torch.tensor([1.0]))[:, 0].tolist() == [6.0, 54.0, 533.0]


def test_delta_rule_overwrites_what_a_key_held():
    """With beta 1 and no decay a key written twice holds its second value, and another key's value stays."""
    k = torch.eye(3, dtype=torch.float64)
    S = torch.zeros(3, 2, dtype=torch.float64)
    for key, val in ((0, [1.0, 2.0]), (1, [5.0, 6.0]), (0, [7.0, 8.0])):
        u = torch.tensor(val, dtype=torch.float64) - S.T @ k[key]
        S = S + torch.outer(k[key], u)
    assert (S.T @ k[0]).tolist() == [7.0, 8.0] and (S.T @ k[1]).tolist() == [5.0, 6.0]


def test_cap_sink_and_chunk():
    s = torch.tensor([0.01, 100.0, -100.0], dtype=torch.float64)
    c = P.capped(s, 5.0)
    assert abs(float(c[0]) - 0.01) < 1e-6 and abs(float(c[1]) - 5.0) < 1e-9 and abs(float(c[2]) + 5.0) < 1e-9
    assert P.capped(s, None) is s
    assert [j for j in range(12) if P.sees(9, j, 4)] == [8, 9] and [j for j in range(12) if P.sees(7, j, 4)] == [4, 5, 6, 7]
    assert [j for j in range(12) if P.sees(3, j, None)] == [0, 1, 2, 3]
    # one token alone: its score is cap * tanh(...), its weight e^s / (e^s + e^sink)
    m = _attn(1, 1, 4, 4, 4, 0, softcap=2.0, scale=3.0)
    W = {"q": torch.eye(4, dtype=torch.float64), "k": torch.eye(4, dtype=torch.float64), "v": torch.eye(4, dtype=torch.float64),
         "o": torch.eye(4, dtype=torch.float64), "sink": torch.tensor([0.7], dtype=torch.float64)}
    h = torch.tensor([[1.0, 2.0, 3.0, 4.0]], dtype=torch.float64)
    e = math.exp(2.0 * math.tanh(4.0 * 3.0 / 2.0))                            # normed q . k = 4
    assert torch.allclose(P.attention(h, [0], W, "", m, 0.0), h * e / (e + math.exp(0.7)))


@pytest.mark.parametrize("kind,mixer,unseen", [("attention", _attn(2, 1, 8, 6, 4, 4), 7), ("delta", _delta(2, 1, 8, 6, 3), None),
                                                ("mamba1", _mamba(12, 3, 2, 2), None)])
def test_what_a_position_depends_on(kind, mixer, unseen):
    """One layer at position 10: tokens behind it and in another chunk change nothing, tokens in sight do; the recurrent
    mixers remember the first token."""
    cfg = one_layer(kind, mixer, width=16)
    W = _weights(cfg)
    torch.manual_seed(0)
    h = torch.randn(12, 16, dtype=torch.float64)
    base = P.mixer(kind, h, list(range(12)), W, "l0.mix.", mixer, 1e-6)[10]
    for j, seen in ((11, False), (unseen, False), (8, True), (0, unseen is None)):
        if j is None:
            continue
        h2 = h.clone()
        h2[j] += 1.0
        moved = P.mixer(kind, h2, list(range(12)), W, "l0.mix.", mixer, 1e-6)[10]
        assert (not torch.equal(moved, base)) == seen, f"{kind}: position {j}"


def test_a_layer_on_another_layers_weights_is_a_layer_of_its_own():
    mixer = _delta(1, 1, 4, 4, 2)
    cfg = one_layer("delta", mixer, 8, width=16)
    twice = copy.deepcopy(cfg)
    twice["layers"].append(_layer("delta", mixer, 8, weights_of=0))
    W = _weights(cfg)
    stream = []
    P.forward(twice, W, [1, 2, 3], stream)
    doubled = {**W, **{n.replace("l0.", "l1.", 1): t for n, t in W.items() if n.startswith("l0.")}}
    unshared = copy.deepcopy(twice)
    unshared["layers"][1].pop("weights_of")
    stream2 = []
    P.forward(unshared, doubled, [1, 2, 3], stream2)
    assert torch.equal(stream[1], stream2[1]) and not torch.equal(stream[0], stream[1])
    assert set(_model(twice).tensor_decls()) == set(W)
