"""Shared by the Vubotar tests: small configurations (none of them a real model's sizes) and random weights for the
framework and for the plain implementation alike."""
from __future__ import annotations

import copy

import torch

from tensorline_amd.config.vubotar_config import VubotarConfig


def _latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, base=500.0, scale=None):
    return {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
            "scale": scale if scale is not None else (dim + rot_dim) ** -0.5, "rot": {"base": base, "dims": rot_dim}}


def _attn(heads, kv_heads, dim, vdim, window, keep_first=0, bias_max=40, rows=12, softcap=9.0, scale=None, v_mix=True):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5,
         "bias_max": bias_max, "bias_rows": rows, "v_mix": v_mix}
    if softcap:
        m["softcap"] = softcap
    if window:
        m["mask"] = {"size": window}
        if keep_first:
            m["mask"]["keep_first"] = keep_first
    return m


def _mlstm(heads, dim, vdim, cap=7.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}


def _moe(experts, top, ff):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def _layer(kind, mixer, mlp=None):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def _model(vocab, width, layers, eps=1e-5, scale=2.0, logit_scale=0.6, cap=11.0):
    out = {"architecture": "Vubotar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
           "logit_scale": logit_scale, "layers": layers}
    if cap:
        out["logit_softcap"] = cap
    return out


# all three mixers, a layer without feed-forward, three layers that share values, one between them that does not, value sizes
# above and below the key sizes, a window on neither a page's nor a tile's border
CFG_A = _model(320, 96, [
    _layer("mlstm", _mlstm(2, 24, 40), _moe(6, 2, 40)),
    _layer("attention", _attn(4, 2, 24, 40, 21, 3), _moe(8, 3, 24)),
    _layer("latent_attention", _latent(3, 16, 8, 24, 20, 40), _moe(5, 2, 40)),
    _layer("attention", _attn(4, 2, 16, 24, 33, 17, bias_max=25, rows=16, softcap=3.0, v_mix=False)),
    _layer("attention", _attn(2, 2, 40, 40, 37, 5, bias_max=70, rows=9), _moe(6, 2, 40)),
    _layer("mlstm", _mlstm(3, 40, 16, 12.0)),
    _layer("attention", _attn(8, 4, 24, 20, 21, 3, bias_max=9, rows=8, softcap=25.0), _moe(4, 4, 16)),
])
# sizes that are no multiple of 8, one head, a table of two rows, a window wider than any prompt, no window, nothing capped,
# as many choices as experts, one expert, a latent of one column, factors of one
CFG_B = _model(131, 72, [
    _layer("latent_attention", _latent(1, 6, 2, 9, 1, 11, base=50.0), _moe(3, 3, 20)),
    _layer("attention", _attn(3, 1, 10, 7, 500, bias_max=3, rows=2, softcap=None, scale=0.4), _moe(1, 1, 16)),
    _layer("mlstm", _mlstm(1, 7, 9, 2.0), _moe(2, 1, 9)),
    _layer("attention", _attn(1, 1, 6, 7, 0, bias_max=200, rows=31, softcap=4.0)),
    _layer("attention", _attn(7, 1, 20, 7, 1, 2, bias_max=5, rows=5)),
    _layer("latent_attention", _latent(3, 4, 4, 6, 9, 30)),
], eps=1e-6, scale=1.0, logit_scale=1.0, cap=None)
# head sizes the bfloat16 matrix-core attention takes, more kept first tokens than a page holds, key sizes of 64 and 128, a
# cached row of 256
CFG_C = _model(200, 128, [
    _layer("attention", _attn(6, 1, 64, 64, 40, 20, bias_max=30, rows=10), _moe(8, 2, 16)),
    _layer("mlstm", _mlstm(1, 128, 72), _moe(5, 1, 48)),
    _layer("latent_attention", _latent(4, 32, 16, 32, 24, 136), _moe(6, 3, 32)),
    _layer("attention", _attn(2, 1, 128, 64, 100, 2, bias_max=64, rows=20, softcap=30.0, scale=0.05)),
    _layer("mlstm", _mlstm(4, 64, 144), _moe(3, 2, 24)),
    _layer("attention", _attn(4, 2, 32, 32, 70, 0, bias_max=300, rows=32, v_mix=True)),
], scale=4.0, logit_scale=0.3, cap=20.0)
CONFIGS = {"A": CFG_A, "B": CFG_B, "C": CFG_C}


def one_layer(kind: str, mixer: dict, mlp=None, width: int = 64, vocab: int = 50) -> dict:
    return _model(vocab, width, [_layer(kind, mixer, mlp)], eps=1e-6)


def typed(cfg: dict) -> VubotarConfig:
    return VubotarConfig.from_dict(copy.deepcopy(cfg))


def spread(w: dict) -> None:
    """Random weights that keep every mechanism in play: matrices scaled to their inputs, so that gates and scores spread over
    their ranges, forget gates that keep dozens of tokens.  Queries of a matrix memory lean towards their keys: its output is a
    quotient whose denominator n . q would else pass through zero now and then, where no arithmetic keeps its digits."""
    for name, t in w.items():
        if t.dim() == 2 and name not in ("embed",) and not name.endswith(".rel"):
            t.mul_(0.8 / (float(t.std()) + 1e-9) / t.shape[1] ** 0.5)
        if name.endswith("f.b"):
            t.add_(3.0)
        if name.endswith(".rel"):
            t.mul_(1.5)
        if name.endswith(".correction"):
            t.mul_(15.0)
    for name in [n for n in w if n.endswith("mix.i.b")]:
        q, k = w[name[:-3] + "q"], w[name[:-3] + "k"]
        q.mul_(0.5).add_(k)
    if "embed" in w:
        w["embed"].mul_(25.0)


def build(cfg: dict, dtype: str, seed: int = 0, device="cuda:0", edit=spread):
    """(framework model, plain weights by name in float32).  Both hold the same bfloat16-rounded
    values; ``edit(weights)`` changes them first (the model is then loaded from the edited ones)."""
    from tensorline_amd.config.registry import get_architecture
    from tensorline_amd.engine.loading import TORCH_DTYPE
    from tensorline_amd.models.decoder import DecoderModel
    from tensorline_amd.weights.loader import load_from_getter
    from tensorline_amd.weights.random_init import random_tensor
    config = typed(cfg)
    model = DecoderModel(get_architecture("Vubotar").build_spec(config), TORCH_DTYPE[dtype], device)
    w = {name: random_tensor(name, decl, seed, "cpu") for name, decl in model.tensor_decls().items()}
    if edit is not None:
        edit(w)
        for name in w:
            w[name] = w[name].to(torch.bfloat16).to(torch.float32)
    load_from_getter(model, lambda name, decl: w[name], device)
    return model, w


def routed_layers(cfg: dict) -> list[int]:
    return [i for i, layer in enumerate(cfg["layers"]) if layer.get("mlp") is not None]


def random_config(rng) -> dict:
    """A configuration drawn from ``rng`` (a ``random.Random``): one to six layers of the three kinds in any order, sizes that
    are and are not multiples of 8 or 16, every head grouping, windows, kept first tokens and reaches from one token to more
    than a prompt, layers that share values and layers that do not."""
    def divisor(n):
        return rng.choice([d for d in range(1, n + 1) if n % d == 0])

    values = rng.choice([(1, 4), (2, 12), (4, 8), (2, 32), (1, 64), (4, 16)])       # kv_heads, vdim of the first mixing layer
    layers = []
    for _ in range(rng.randint(1, 6)):
        kind = rng.choice(["mlstm", "latent_attention", "attention", "attention"])
        heads = rng.choice([1, 2, 3, 4, 6, 8])
        if kind == "mlstm":
            m = _mlstm(heads, rng.choice([4, 7, 16, 24, 32, 40, 64, 96, 128, 130]), rng.choice([4, 9, 16, 24, 32, 64, 80]), rng.choice([1.5, 7.0, 15.0]))
        elif kind == "latent_attention":
            m = _latent(heads, rng.choice([4, 8, 16, 24, 32]), rng.choice([2, 4, 8, 16]), rng.choice([4, 8, 12, 32]), rng.choice([1, 5, 16, 33, 64]),
                        rng.choice([5, 16, 40, 100, 200]), base=rng.choice([50.0, 10000.0]), scale=rng.choice([0.05, 0.125, 0.3]))
        else:
            kv, vdim = values
            mix = rng.random() < 0.7
            if not mix:
                kv, vdim = divisor(heads), rng.choice([4, 8, 12, 16, 32, 48, 64, 128])
            rows = rng.choice([2, 3, 8, 15, 32])
            m = _attn(kv * rng.choice([1, 2, 3, 7]), kv, rng.choice([4, 8, 16, 20, 24, 32, 40, 64, 128]), vdim,
                      rng.choice([0, 1, 2, 5, 16, 17, 31, 48, 70, 400]), rng.choice([0, 0, 1, 3, 16, 21]),
                      bias_max=rows // 2 + rng.choice([1, 2, 7, 30, 128, 500]), rows=rows, softcap=rng.choice([None, 2.0, 15.0, 50.0]),
                      scale=rng.choice([0.05, 0.125, 0.3]), v_mix=mix)
        experts = rng.randint(1, 9)
        layers.append(_layer(kind, m, rng.choice([None, _moe(experts, rng.randint(1, experts), rng.choice([8, 20, 36, 64]))])))
    return _model(rng.randint(50, 400), rng.choice([24, 36, 50, 64, 72, 100, 128, 200]), layers, eps=rng.choice([1e-5, 1e-6]),
                  scale=rng.choice([1.0, 3.5]), logit_scale=rng.choice([0.2, 1.0]), cap=rng.choice([None, 5.0, 30.0]))
