"""Vubotar without a GPU: the configuration reader and what it refuses, the size read from a tensor's shape, the spec (mixer
kinds, cache and state needs, tensor names), the buckets of distances, and pins of the plain implementation
(tests/plain_vubotar.py) against closed forms."""
import copy
import math

import pytest
import torch

from tensorline_amd.config.model_config import ConfigError
from tensorline_amd.config.registry import get_architecture, known_architectures, load_model_config
from tensorline_amd.models.decoder import DecoderModel
from tensorline_amd.ops import kernels
from tensorline_amd.parts.masked_attention import distance_buckets
from tensorline_amd.weights.random_init import random_tensor, write_random_model
from tests import plain_vubotar as P
from tests.vubotar_helpers import CFG_A, CFG_B, CFG_C, _attn, _latent, _mlstm, _moe, one_layer, typed

F = torch.float64


def _model(cfg):
    return DecoderModel(get_architecture("Vubotar").build_spec(typed(cfg)), torch.float32, "cpu")


def _weights(cfg, seed=0):
    return {n: random_tensor(n, d, seed, "cpu").to(F) for n, d in _model(cfg).tensor_decls().items()}


def test_registered_and_round_trips():
    assert "Vubotar" in known_architectures()
    for cfg in (CFG_A, CFG_B, CFG_C):
        t = typed(cfg)
        assert typed(t.to_dict()) == t


@pytest.mark.parametrize("edit, text", [
    (lambda c: c["layers"][0].update(type="slstm"), "unknown"),
    (lambda c: c["layers"][0].pop("mixer"), "mixer is missing"),
    (lambda c: c["layers"][0]["mixer"].pop("gate_cap"), "gate_cap must be"),
    (lambda c: c["layers"][0]["mixer"].update(gate_cap=0.0), "gate_cap must be"),
    (lambda c: c["layers"][0]["mixer"].update(dim=0), "dim must be"),
    (lambda c: c["layers"][1]["mixer"].update(heads=3), "not a multiple"),
    (lambda c: c["layers"][1]["mixer"].pop("scale"), "scale must be"),
    (lambda c: c["layers"][1]["mixer"].pop("bias_max"), "bias_max must be"),
    (lambda c: c["layers"][1]["mixer"].update(bias_max=6), "do not fit"),
    (lambda c: c["layers"][1]["mixer"].update(softcap=-1.0), "softcap must be"),
    (lambda c: c["layers"][1]["mixer"]["mask"].update(size=0), "size must be"),
    (lambda c: c["layers"][1]["mixer"]["mask"].update(keep_first=-1), "keep_first"),
    (lambda c: c["layers"][4]["mixer"].update(vdim=16), "another size"),
    (lambda c: c["layers"][2]["mixer"].pop("q_rank"), "q_rank must be"),
    (lambda c: c["layers"][2]["mixer"]["rot"].update(dims=4), "equal rot_dim"),
    (lambda c: c["layers"][2]["mixer"].pop("rot"), "dims must be"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "unknown"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=7), "exceeds"),
    (lambda c: c.update(logit_softcap=0), "logit_softcap must be"),
    (lambda c: c.pop("norm"), "norm.eps"),
])
def test_reader_refuses(edit, text):
    cfg = copy.deepcopy(CFG_A)
    edit(cfg)
    with pytest.raises(ConfigError, match=text):
        typed(cfg)


def test_rows_of_the_distance_table_come_from_the_checkpoint(tmp_path):
    import json
    folder = write_random_model(typed(CFG_B), str(tmp_path / "m"), seed=2)
    raw = json.loads((tmp_path / "m" / "config.json").read_text())
    for layer in raw["layers"]:
        layer["mixer"].pop("bias_rows", None)
    (tmp_path / "m" / "config.json").write_text(json.dumps(raw))
    arch, cfg = load_model_config(folder)
    assert [l["mixer"].get("bias_rows") for l in cfg.layers] == [None, 2, None, 31, 5, None]
    assert cfg == typed(CFG_B) and arch.name == "Vubotar"


def test_spec_kinds_needs_and_names():
    m = _model(CFG_A)
    assert [type(b.mixer).__name__ for b in m.blocks] == ["MatrixLSTM", "MaskedAttention", "LatentAttention", "MaskedAttention",
                                                          "MaskedAttention", "MatrixLSTM", "MaskedAttention"]
    assert [getattr(b.mixer, "value_mix", None) for b in m.blocks] == [None, "first", None, None, "mix", None, "mix"]
    states, caches = m.state_needs(), m.cache_needs()
    # S of every head, then a copy of n and m per 16 value columns
    assert states[0].shape == (2 * (40 * 24 + 3 * 25),) and states[5].shape == (3 * (16 * 40 + 1 * 41),) and states[1] is None
    assert [(c.window, c.keep_first) if c else None for c in caches] == [None, (21, 3), (0, 0), (33, 17), (37, 5), None, (21, 3)]
    assert caches[1].planes[0].shape == (2, 48) and caches[2].planes[0].shape == (1, 64)
    decls = m.tensor_decls()
    names = set(decls)
    assert {"embed", "head", "final.norm", "l0.norm1", "l0.norm2", "l0.ls1", "l0.ls2", "l0.mix.i.b", "l0.mix.f.b", "l0.mix.norm",
            "l1.mix.q.norm", "l1.mix.rel", "l1.mix.vmix", "l2.mix.dq", "l2.mix.dq.norm", "l2.mix.uq", "l2.mix.dkv.norm", "l2.mix.g",
            "l1.mlp.e7.down", "l1.mlp.correction", "l1.mlp.router"} <= names
    assert not names & {"l3.mix.vmix", "l3.norm2", "l3.ls2", "l2.mix.q", "l1.mix.sink", "l1.mix.g"}
    assert decls["l1.mix.rel"].shape == (12, 4) and decls["l1.mix.vmix"].shape == () and decls["l2.mix.uq"].shape == (3 * 24, 20)
    assert decls["l2.mix.dkv"].shape == (48, 96) and decls["l0.mix.i"].shape == (2, 96) and decls["head"].shape == (320, 96)


def test_a_layers_values_need_one_that_leaves_them():
    from tensorline_amd.parts.masked_attention import MaskedAttention
    with pytest.raises(ValueError, match="value_mix"):
        MaskedAttention(32, "m.", torch.float32, "cpu", heads=1, kv_heads=1, dim=8, scale=1.0, values="keys", value_mix="mix")
    with pytest.raises(ValueError, match="sink"):
        MaskedAttention(32, "m.", torch.float32, "cpu", heads=1, kv_heads=1, dim=8, scale=1.0, sink="two")
    with pytest.raises(ValueError, match="reach"):
        MaskedAttention(32, "m.", torch.float32, "cpu", heads=1, kv_heads=1, dim=8, scale=1.0, distance_bias={"rows": 8, "reach": 4})


@pytest.mark.parametrize("rows,reach", [(12, 40), (2, 3), (31, 200), (8, 9), (16, 128), (32, 128), (16, 64), (9, 5), (64, 5000), (10, 80), (3, 2)])
def test_buckets_of_distances(rows, reach):
    got = distance_buckets(rows, reach).tolist()
    assert got == [P.bucket(n, rows, reach) for n in range(reach + 1)]
    assert got[-1] == rows - 1 and P.bucket(10 * reach, rows, reach) == rows - 1 and got == sorted(got)
    assert got[:rows // 2] == list(range(rows // 2))


# ---- pins of the plain implementation ---------------------------------------------------------------------
def test_buckets_at_powers():
    # half of 16 rows is 8, and 8 more rows cover 8 .. 128, a factor of sqrt(2) each: two rows to every doubling
    assert [P.bucket(n, 16, 128) for n in (7, 8, 11, 12, 16, 22, 23, 32, 64, 90, 91, 127, 128, 4000)] == [7, 8, 8, 9, 10, 10, 11, 12, 14, 14, 15, 15, 15, 15]


def test_rotation_turns_neighbours_and_leaves_the_rest():
    x = torch.arange(1.0, 7.0, dtype=F).view(1, 6).repeat(2, 1)
    got = P.turn_pairs(x, [0, 3], 4, 16.0)
    assert torch.equal(got[0], x[0])
    a, b = 3.0, 3.0 / 4.0                                  # frequencies 1 and 16^(-2/4)
    want = [math.cos(a) - 2 * math.sin(a), 2 * math.cos(a) + math.sin(a), 3 * math.cos(b) - 4 * math.sin(b), 4 * math.cos(b) + 3 * math.sin(b), 5, 6]
    assert torch.allclose(got[1], torch.tensor(want, dtype=F))


def test_who_sees_whom():
    m = {"size": 3, "keep_first": 2}
    assert [j for j in range(12) if P.sees(9, j, m)] == [0, 1, 7, 8, 9] and [j for j in range(12) if P.sees(3, j, m)] == [0, 1, 2, 3]
    assert [j for j in range(12) if P.sees(5, j, {"size": 1})] == [5] and [j for j in range(4) if P.sees(2, j, None)] == [0, 1, 2]


def test_a_one_in_the_denominator_and_the_order_of_cap_and_bias():
    s = torch.tensor([[0.0, math.log(2.0), 9.0]], dtype=F)
    seen = torch.tensor([[True, True, False]])
    assert torch.allclose(P.attention_weights(s, seen, True), torch.tensor([[0.25, 0.5, 0.0]], dtype=F))
    assert torch.allclose(P.attention_weights(s, seen, False), torch.tensor([[1 / 3, 2 / 3, 0.0]], dtype=F))
    assert torch.allclose(P.attention_weights(s - 1000.0, seen, True), torch.zeros(1, 3, dtype=F))
    # one token alone: its score is cap tanh(4 scale / cap) + rel[0], its weight e^s / (1 + e^s)
    m = _attn(1, 1, 4, 4, 4, bias_max=3, rows=2, softcap=2.0, scale=3.0)
    eye = torch.eye(4, dtype=F)
    W = {"q": eye, "k": eye, "v": eye, "o": eye, "q.norm": torch.ones(4, dtype=F), "k.norm": torch.ones(4, dtype=F),
         "rel": torch.tensor([[0.7], [5.0]], dtype=F)}
    h = torch.tensor([[1.0, 2.0, 3.0, 4.0]], dtype=F)
    e = math.exp(2.0 * math.tanh(4.0 * 3.0 / 2.0) + 0.7)
    assert torch.allclose(P.mixer_attention(h, [0], W, "", m, 0.0), h * e / (1 + e))


def test_values_mixed_with_the_first_layers():
    m = _attn(1, 1, 4, 4, 4)
    W = {"v": 2.0 * torch.eye(4, dtype=F), "vmix": torch.tensor(0.25, dtype=F)}
    h, first = torch.ones(3, 4, dtype=F), 10.0 * torch.ones(3, 4, dtype=F)
    assert torch.allclose(P.attention_values(h, W, "", m, first), 0.75 * 2.0 * h + 2.5)
    assert torch.allclose(P.attention_values(h, W, "", m, None), 2.0 * h)
    assert torch.allclose(P.attention_values(h, W, "", {**m, "v_mix": False}, first), 2.0 * h)


def test_matrix_memory_against_its_closed_form():
    """o_t is a weighted sum of values with weights exp(sum of forget gates + input gate) (q . k); the running maximum and its
    start at zero only set the floor of the denominator."""
    torch.manual_seed(0)
    T, d, dv = 9, 5, 3
    q, k, v = torch.randn(T, d, dtype=F), torch.randn(T, d, dtype=F), torch.randn(T, dv, dtype=F)
    i, f = torch.randn(T, dtype=F) * 3, -torch.rand(T, dtype=F) * 2
    got = P.mlstm_walk(q, k, v, i, f)
    m = 0.0
    for t in range(T):
        m = max(float(f[t]) + m, float(i[t]))
        w = torch.stack([torch.exp(f[s + 1:t + 1].sum() + i[s]) * (q[t] @ k[s]) for s in range(t + 1)])
        scale = math.exp(-m)
        den = max(abs(float(w.sum())) * scale, scale) + 1e-6
        assert torch.allclose(got[t], (w[:, None] * v[:t + 1]).sum(0) * scale / den)
    # nothing written yet worth reading: the floor exp(-m) with m held at zero or above by the start
    tiny = P.mlstm_walk(q[:1], k[:1], v[:1], torch.tensor([-30.0], dtype=F), torch.tensor([-0.1], dtype=F))
    assert float(tiny.abs().max()) < 1e-10


def test_gates():
    W = {"i": torch.zeros(1, 2, dtype=F), "i.b": torch.tensor([100.0], dtype=F), "f": torch.zeros(1, 2, dtype=F), "f.b": torch.tensor([0.0], dtype=F)}
    i, f = P.mlstm_gates(torch.ones(1, 2, dtype=F), W, "", 7.0)
    assert abs(float(i) - 7.0) < 1e-9 and abs(float(f) - math.log(0.5)) < 1e-12
    assert abs(P.log_sigmoid(-50.0) + 50.0) < 1e-12 and abs(P.log_sigmoid(50.0)) < 1e-20


def test_router_chooses_by_corrected_scores_and_weights_by_plain_ones():
    z = torch.tensor([2.0, 0.0, 1.0, -1.0], dtype=F)
    s = torch.sigmoid(z)
    chosen, weights = P.route(z, torch.tensor([-1.0, 0.0, 0.0, 0.9], dtype=F), 2)
    assert chosen == [3, 2]
    assert weights == [float(s[3] / (s[3] + s[2])), float(s[2] / (s[3] + s[2]))]
    assert P.route(z, torch.zeros(4, dtype=F), 2)[0] == [0, 2] and P.route(torch.zeros(4), torch.zeros(4), 2)[0] == [0, 1]
    assert P.is_close_call(z, torch.zeros(4, dtype=F), [0, 1], _moe(4, 2, 8), 0.6) and not P.is_close_call(z, torch.zeros(4, dtype=F), [0, 1], _moe(4, 2, 8), 0.3)


def test_both_branches_read_the_same_stream():
    """With a feed-forward that gives nothing the mixer's branch is alone; the feed-forward reads the stream as the mixer found
    it, so a change of the mixer's factor does not reach it within the layer."""
    cfg = one_layer("mlstm", _mlstm(1, 4, 6), _moe(2, 1, 8), width=16)
    W = _weights(cfg)
    x = W["embed"][torch.tensor([3, 1, 4])] * cfg["embedding"]["scale"]
    stream = lambda w: P.forward(cfg, w, [3, 1, 4], want_layers=True)[1][0]
    full, no_mixer, no_ff = stream(W), stream({**W, "l0.ls1": torch.zeros(16, dtype=F)}), stream({**W, "l0.ls2": torch.zeros(16, dtype=F)})
    assert torch.allclose(full - x, (no_mixer - x) + (no_ff - x), atol=1e-14) and not torch.allclose(no_mixer, x)


@pytest.mark.parametrize("kind,mixer,unseen", [("attention", _attn(2, 1, 8, 6, 4, 2, rows=4), 4), ("latent_attention", _latent(2, 8, 4, 6, 7, 9), None),
                                                ("mlstm", _mlstm(2, 6, 5), None)])
def test_what_a_position_depends_on(kind, mixer, unseen):
    """One layer at position 10: tokens behind it and between the kept first ones and the window change nothing, tokens in sight
    do; the other mixers remember the first token."""
    cfg = one_layer(kind, mixer, width=16)
    W = _weights(cfg)
    torch.manual_seed(0)
    h = torch.randn(12, 16, dtype=F)
    base = P.mixer(kind, h, list(range(12)), W, "l0.mix.", mixer, 1e-6)[10]
    for j, seen in ((11, False), (unseen, False), (8, True), (0, True), (1, True)):
        if j is None:
            continue
        h2 = h.clone()
        h2[j] += 1.0
        moved = P.mixer(kind, h2, list(range(12)), W, "l0.mix.", mixer, 1e-6)[10]
        assert (not torch.equal(moved, base)) == seen, f"{kind}: position {j}"


def test_state_layout_covers_every_block_of_value_columns():
    assert kernels.matrix_lstm_state(1, 8, 16) == 16 * 8 + 9
    assert kernels.matrix_lstm_state(3, 8, 17) == 3 * (17 * 8 + 2 * 9)
