"""``Taluvik``: how its configuration turns into layers and the order they run in.

A decoder whose layers have one layer norm (weight and bias) ahead of two branches that run side by side: ``h =
norm1(x)``, ``x <- x + m (mixer(h) + ff(h))``.  Each layer has one of three mixers:

* ``delta``: the gated delta rule behind short convolutions, with unit queries and keys;
* ``mamba1``: Mamba's selective scan;
* ``attention``: grouped heads; part of a head turned in halves by frequencies stretched in wavelength bands; queries and
  keys divided by their root mean square per head; scores bent by a cap; a token sees its own chunk of positions up to
  itself; a learned sink per head in the softmax's denominator.

Feed-forwards are ``W_down (gelu_tanh(W_gate h) * W_up h)`` or absent.  A layer may run on another layer's weights
(``weights_of``) and keeps its own cache or state: the schedule names that layer again.  Embedding rows enter times
``embedding.scale``; the head is a matrix of its own behind a final layer norm.  Tensor names: ``embed``, ``l<i>.norm1``
(``.b``), ``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm`` (``.b``), ``head``.
"""
from __future__ import annotations

from tensorline_amd.config.registry import Architecture, register_architecture
from tensorline_amd.config.taluvik_config import TaluvikConfig
from tensorline_amd.parts.spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry


def _mixer(cfg: TaluvikConfig, layer: dict) -> PartSpec:
    m, kind = layer["mixer"], layer["type"]
    if kind == "delta":
        return PartSpec("gated_delta", {"heads": m["heads"], "kv_heads": m["kv_heads"], "dim": m["dim"], "vdim": m["vdim"],
                                        "conv": m["conv"], "eps": cfg.norm_eps, "unit_eps": 1e-6}, prefix="mix.")
    if kind == "mamba1":
        return PartSpec("selective_scan", {"inner": m["inner"], "state": m["state"], "dt_rank": m["dt_rank"], "conv": m["conv"]},
                        prefix="mix.")
    mask, rot = m.get("mask"), m.get("rot")
    return PartSpec("masked_attention", {
        "heads": m["heads"], "kv_heads": m["kv_heads"], "dim": m["dim"], "vdim": m["vdim"], "scale": m["scale"], "values": "proj",
        "mask": {"kind": "chunk", "size": mask["size"]} if mask else None, "qk_norm": "plain", "eps": cfg.norm_eps,
        "rot": {**rot, "layout": "halves"} if rot else None, "softcap": m.get("softcap"), "sink": True}, prefix="mix.")


def _feed_forward(mlp: dict | None) -> PartSpec | None:
    if mlp is None:
        return None
    return PartSpec("swiglu", {"intermediate_size": mlp["ff"], "names": ("gate", "up", "down"), "activation": "gelu_tanh"},
                    prefix="mlp.")


def taluvik_spec(cfg: TaluvikConfig) -> ModelSpec:
    norm = lambda name: PartSpec("layernorm", {"eps": cfg.norm_eps, "name": name})
    owners = [cfg.weight_layer(i) for i in range(len(cfg.layers))]
    layers, index = [], {}                    # a layer is built once per set of tensors
    for i, layer in enumerate(cfg.layers):
        if owners[i] != i:
            continue
        index[i] = len(layers)
        layers.append(LayerSpec(prefix=f"l{i}.", mixer=_mixer(cfg, layer), feed_forward=_feed_forward(layer.get("mlp")),
                                mixer_norm=norm("norm1"), feed_forward_norm=None, block="parallel_branches",
                                branch_scale=cfg.residual_mult))
    spec = ModelSpec(
        hidden_size=cfg.hidden_size, vocab_size=cfg.vocab_size,
        embedding=PartSpec("token_embedding", {"name": "embed", "scale": cfg.embedding_scale}),
        layers=tuple(layers), final_norm=norm("final.norm"), head=PartSpec("lm_head", {"name": "head"}),
        schedule=tuple(ScheduleEntry(index[j]) for j in owners),
        max_position=cfg.max_position_embeddings, eos_token_ids=tuple(cfg.eos_token_id))
    spec.validate()
    return spec


TALUVIK = register_architecture(Architecture("Taluvik", TaluvikConfig, taluvik_spec), replace=True)
