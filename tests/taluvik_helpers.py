"""Shared by the Taluvik tests: small configurations (none of them a real model's sizes) and random weights for the
framework and for the plain implementation alike."""
from __future__ import annotations

import copy

import torch

from tensorline_amd.config.taluvik_config import TaluvikConfig

BANDS = {"factor": 3.0, "low": 1.5, "high": 5.0, "original": 100}


def _delta(heads, kv_heads, dim, vdim, conv=4):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def _mamba(inner, state, rank, conv=4):
    return {"inner": inner, "state": state, "dt_rank": rank, "conv": conv}


def _attn(heads, kv_heads, dim, vdim, chunk, dims, base=500.0, scaling=BANDS, softcap=7.0, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5}
    if softcap:
        m["softcap"] = softcap
    if dims:
        m["rot"] = {"dims": dims, "base": base}
        if scaling:
            m["rot"]["scaling"] = scaling
    if chunk:
        m["mask"] = {"size": chunk}
    return m


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _layer(kind, mixer, ff=None, weights_of=None):
    out = {"type": kind, "mixer": mixer, "mlp": _dense(ff) if ff else None}
    if weights_of is not None:
        out["weights_of"] = weights_of
    return out


def _model(vocab, width, layers, eps=1e-5, scale=6.0, mult=0.6):
    return {"architecture": "Taluvik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "residual_mult": mult, "layers": layers}


# all three mixers, a layer without feed-forward, every mixer run again on the first run's weights, value sizes above and
# below the key sizes, partial and full rotation, a chunk on neither a page's nor a tile's border
_A0, _A1, _A2 = _delta(4, 2, 24, 40), _mamba(88, 12, 8), _attn(4, 2, 24, 40, 19, 8)
CFG_A = _model(320, 96, [
    _layer("delta", _A0, 136), _layer("mamba1", _A1, 64), _layer("attention", _A2, 136), _layer("delta", _delta(2, 2, 40, 16, 3)),
    _layer("mamba1", _A1, 64, weights_of=1), _layer("delta", _A0, 136, weights_of=0), _layer("attention", _A2, 136, weights_of=2),
])
# sizes that are no multiple of 8, one head, one state, a rank of one, a convolution of one tap and one of six, a chunk of
# one page, attention first, a layer that runs three times in a row, no rotation, no cap, factor 1 on the branches
_B0, _B1, _B2 = _attn(3, 1, 10, 7, 16, 0, softcap=None, scale=0.4), _mamba(50, 1, 1, 6), _delta(3, 1, 9, 13, 1)
CFG_B = _model(131, 72, [
    _layer("attention", _B0, 50), _layer("mamba1", _B1), _layer("mamba1", _B1, weights_of=1), _layer("mamba1", _B1, weights_of=1),
    _layer("delta", _B2, 20), _layer("attention", _attn(1, 1, 6, 9, 2, 6, base=50.0, scaling=None), 7), _layer("mamba1", _mamba(36, 20, 5, 2), 16),
], eps=1e-6, scale=1.0, mult=1.0)
# head sizes the bfloat16 matrix-core attention takes, key sizes of 64 and 128, states on two and more lanes, no chunk
CFG_C = _model(200, 128, [
    _layer("attention", _attn(6, 1, 64, 64, 40, 32), 64), _layer("delta", _delta(2, 1, 128, 64, 4), 48), _layer("mamba1", _mamba(144, 40, 16, 3), 32),
    _layer("attention", _attn(2, 2, 128, 96, 0, 128, base=10000.0, scaling=None, softcap=3.0, scale=0.05)), _layer("delta", _delta(4, 4, 64, 128, 2), 64),
    _layer("attention", _attn(4, 2, 32, 32, 70, 16, softcap=20.0), 64),
], scale=11.0, mult=0.4)
CONFIGS = {"A": CFG_A, "B": CFG_B, "C": CFG_C}


def one_layer(kind: str, mixer: dict, ff=None, width: int = 64, vocab: int = 50) -> dict:
    return _model(vocab, width, [_layer(kind, mixer, ff)], eps=1e-6, scale=4.0, mult=0.7)


def typed(cfg: dict) -> TaluvikConfig:
    return TaluvikConfig.from_dict(copy.deepcopy(cfg))


def spread(w: dict) -> None:
    """Random weights that keep every mechanism in play: matrices scaled to their inputs, so that gates, steps and scores
    spread over their ranges; decays from a few tokens to thousands; sinks and biases of the scores' size."""
    for name, t in w.items():
        leaf = name.rsplit(".", 1)[-1]
        if t.dim() == 2 and leaf not in ("conv", "A_log") and name != "embed":
            t.mul_(0.7 / (0.02 * t.shape[1] ** 0.5))
        if name.endswith("dt_bias") or name.endswith("dt.b"):
            t.sub_(3.0)
        if name.endswith("sink"):
            t.mul_(1.5)
    if "embed" in w:
        w["embed"].mul_(8.0)


def build(cfg: dict, dtype: str, seed: int = 0, device="cuda:0", edit=spread):
    """(framework model, plain weights by name in float32).  Both hold the same bfloat16-rounded
    values; ``edit(weights)`` changes them first (the model is then loaded from the edited ones)."""
    from tensorline_amd.config.registry import get_architecture
    from tensorline_amd.engine.loading import TORCH_DTYPE
    from tensorline_amd.models.decoder import DecoderModel
    from tensorline_amd.weights.loader import load_from_getter
    from tensorline_amd.weights.random_init import random_tensor
    config = typed(cfg)
    model = DecoderModel(get_architecture("Taluvik").build_spec(config), TORCH_DTYPE[dtype], device)
    w = {name: random_tensor(name, decl, seed, "cpu") for name, decl in model.tensor_decls().items()}
    if edit is not None:
        edit(w)
        for name in w:
            w[name] = w[name].to(torch.bfloat16).to(torch.float32)
    load_from_getter(model, lambda name, decl: w[name], device)
    return model, w


def random_config(rng) -> dict:
    """A configuration drawn from ``rng`` (a ``random.Random``): one to six layers of the three kinds in any order, some run
    again, sizes that are and are not multiples of 8 or 16, every head grouping, chunks from one token to more than a prompt."""
    def divisor(n):
        return rng.choice([d for d in range(1, n + 1) if n % d == 0])

    layers = []
    for i in range(rng.randint(1, 6)):
        if layers and rng.random() < 0.3:
            j = rng.randrange(len(layers))
            layers.append({**copy.deepcopy(layers[j]), "weights_of": j})
            continue
        kind = rng.choice(["delta", "mamba1", "attention"])
        ff = rng.choice([None, 7, 24, 50, 136])
        heads = rng.choice([1, 2, 3, 4, 6, 8])
        if kind == "delta":
            m = _delta(heads, divisor(heads), rng.choice([4, 7, 16, 24, 32, 40, 64, 96, 128, 130]), rng.choice([4, 9, 16, 24, 32, 64, 80]),
                       rng.choice([1, 2, 3, 4, 5]))
        elif kind == "mamba1":
            m = _mamba(rng.choice([16, 30, 64, 100, 200]), rng.choice([1, 4, 8, 12, 16, 17, 32, 40, 100]), rng.choice([1, 4, 5, 8, 16]),
                       rng.choice([1, 2, 3, 4, 7]))
        else:
            dim = rng.choice([4, 8, 16, 20, 24, 32, 40, 64, 128])
            dims = rng.choice([0] + [d for d in (2, 4, 8, 16, 32, 64, 128) if d <= dim])
            m = _attn(heads, divisor(heads), dim, rng.choice([4, 8, 12, 16, 32, 48, 64, 128]), rng.choice([0, 1, 2, 5, 16, 17, 31, 48, 70, 400]),
                      dims, base=rng.choice([50.0, 10000.0]), scaling=rng.choice([None, BANDS, {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 40}]),
                      softcap=rng.choice([None, 2.0, 15.0]), scale=rng.choice([0.05, 0.125, 0.3]))
        layers.append(_layer(kind, m, ff))
    return _model(rng.randint(50, 400), rng.choice([24, 36, 50, 64, 72, 100, 128, 200]), layers, eps=rng.choice([1e-5, 1e-6]),
                  scale=rng.choice([1.0, 5.5]), mult=rng.choice([0.25, 1.0]))
