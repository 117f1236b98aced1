"""Typed configuration of the Vubotar decoder: layers of three kinds of mixers beside routed experts, each branch behind a
norm of its own.

``config.json`` gives: ``architecture`` "Vubotar", ``vocab``, ``width``, ``norm.eps``, ``embedding.scale``, ``logit_scale``,
``logit_softcap`` and ``layers``, one entry per layer: ``type`` and ``mixer``,

* "latent_attention": {heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, rot {dims, base}};
* "attention": {heads, kv_heads, dim, vdim, scale, softcap?, bias_max, mask {size, keep_first?}?, v_mix?};
* "mlstm": {heads, dim, vdim, gate_cap};

and ``mlp`` = {kind "moe", router {experts, top}, expert {ff}} or null.  The rows of an attention layer's distance table are
only a tensor's shape; a configuration without a checkpoint names them ``bias_rows`` in the mixer.
"""
from __future__ import annotations

import copy
import dataclasses
import json
import os
from dataclasses import dataclass, field
from typing import Any, Mapping

from tensorline_amd.config.model_config import ConfigError

LAYER_TYPES = ("latent_attention", "attention", "mlstm")
_INT_KEYS = {"latent_attention": ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank"),
             "attention": ("heads", "kv_heads", "dim", "vdim", "bias_max"),
             "mlstm": ("heads", "dim", "vdim")}


def _positive_int(where: str, d: Any, key: str) -> int:
    v = d.get(key) if isinstance(d, Mapping) else None
    if isinstance(v, bool) or not isinstance(v, int) or v <= 0:
        raise ConfigError(f"config.json: {where}.{key} must be a positive integer, got {v!r}")
    return v


def _number(where: str, d: Any, key: str, positive: bool = False) -> float:
    v = d.get(key) if isinstance(d, Mapping) else None
    if isinstance(v, bool) or not isinstance(v, (int, float)) or (positive and not v > 0.0):
        raise ConfigError(f"config.json: {where}.{key} must be a {'positive ' if positive else ''}number, got {v!r}")
    return float(v)


def _check_attention(where: str, m: Mapping) -> None:
    if m["heads"] % m["kv_heads"]:
        raise ConfigError(f"config.json: {where}: {m['heads']} heads are not a multiple of {m['kv_heads']} kv_heads")
    _number(where, m, "scale", positive=True)
    if m.get("softcap") is not None:
        _number(where, m, "softcap", positive=True)
    if m.get("mask") is not None:
        _positive_int(where + ".mask", m["mask"], "size")
        first = m["mask"].get("keep_first", 0)
        if isinstance(first, bool) or not isinstance(first, int) or first < 0:
            raise ConfigError(f"config.json: {where}.mask.keep_first {first!r} must be a non-negative integer")
    if m.get("bias_rows") is not None:
        rows = _positive_int(where, m, "bias_rows")
        if rows < 2 or m["bias_max"] <= rows // 2:
            raise ConfigError(f"config.json: {where}: a distance table of {rows} rows and a bias_max of {m['bias_max']} do not fit")


def _check_latent(where: str, m: Mapping) -> None:
    _number(where, m, "scale", positive=True)
    rot = m.get("rot")
    if _positive_int(where + ".rot", rot, "dims") != m["rot_dim"] or m["rot_dim"] % 2:
        raise ConfigError(f"config.json: {where}: rot.dims must equal rot_dim and be even")
    _number(where + ".rot", rot, "base", positive=True)


def _check_layer(where: str, layer: Any) -> None:
    if not isinstance(layer, Mapping):
        raise ConfigError(f"config.json: {where} must be an object")
    kind, mixer = layer.get("type"), layer.get("mixer")
    if kind not in LAYER_TYPES:
        raise ConfigError(f"config.json: {where}.type {kind!r} is unknown; known: {', '.join(LAYER_TYPES)}")
    if not isinstance(mixer, Mapping):
        raise ConfigError(f"config.json: {where}.mixer is missing")
    where_m = where + ".mixer"
    for key in _INT_KEYS[kind]:
        _positive_int(where_m, mixer, key)
    if kind == "attention":
        _check_attention(where_m, mixer)
    elif kind == "latent_attention":
        _check_latent(where_m, mixer)
    else:
        _number(where_m, mixer, "gate_cap", positive=True)
    mlp = layer.get("mlp")
    if mlp is not None:
        where += ".mlp"
        if not isinstance(mlp, Mapping) or mlp.get("kind", "moe") != "moe":
            raise ConfigError(f"config.json: {where}.kind {mlp.get('kind') if isinstance(mlp, Mapping) else mlp!r} is unknown; known: moe")
        experts, top = _positive_int(where + ".router", mlp.get("router"), "experts"), _positive_int(where + ".router", mlp.get("router"), "top")
        if top > experts:
            raise ConfigError(f"config.json: {where}.router.top {top} exceeds the {experts} experts")
        _positive_int(where + ".expert", mlp.get("expert"), "ff")


@dataclass(frozen=True)
class VubotarConfig:
    vocab_size: int
    hidden_size: int
    layers: tuple = ()                      # the entries of config.json's ``layers``, checked
    norm_eps: float = 1e-6
    embedding_scale: float = 1.0
    logit_scale: float = 1.0
    logit_softcap: float | None = None
    eos_token_id: tuple[int, ...] = ()
    max_position_embeddings: int = 1 << 30
    architecture: str = "Vubotar"
    extra: Mapping[str, Any] = field(default_factory=dict, compare=False, hash=False)

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    def first_mixing_layer(self) -> int | None:
        """The first attention layer whose values the later ones mix in, or None."""
        return next((i for i, l in enumerate(self.layers) if l["type"] == "attention" and l["mixer"].get("v_mix")), None)

    @classmethod
    def from_dict(cls, d: Mapping[str, Any]) -> "VubotarConfig":
        vocab, width = _positive_int("", d, "vocab"), _positive_int("", d, "width")
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        eps = _number("norm", d.get("norm"), "eps")
        for i, layer in enumerate(layers):
            _check_layer(f"layers[{i}]", layer)
        cap = _number("", d, "logit_softcap", positive=True) if d.get("logit_softcap") is not None else None
        eos = d.get("eos_token_id")
        eos_ids = () if eos is None else tuple(int(e) for e in eos) if isinstance(eos, (list, tuple)) else (int(eos),)
        known = {"architecture", "architectures", "vocab", "width", "layers", "norm", "embedding", "logit_scale", "logit_softcap",
                 "eos_token_id", "max_position_embeddings"}
        out = cls(vocab_size=vocab, hidden_size=width, layers=tuple(copy.deepcopy(dict(l)) for l in layers), norm_eps=eps,
                  embedding_scale=float((d.get("embedding") or {}).get("scale", 1.0)), logit_scale=float(d.get("logit_scale", 1.0)),
                  logit_softcap=cap, eos_token_id=eos_ids, max_position_embeddings=int(d.get("max_position_embeddings", 1 << 30)),
                  extra={k: v for k, v in d.items() if k not in known})
        first = out.first_mixing_layer()
        for i, layer in enumerate(out.layers):
            m = layer["mixer"]
            if layer["type"] == "attention" and m.get("v_mix"):
                want = out.layers[first]["mixer"]
                if m["kv_heads"] * m["vdim"] != want["kv_heads"] * want["vdim"]:
                    raise ConfigError(f"config.json: layers[{i}] mixes in the values of layers[{first}], which are of another size")
        return out

    @classmethod
    def from_json(cls, path: str | os.PathLike) -> "VubotarConfig":
        p = os.fspath(path)
        if os.path.isdir(p):
            p = os.path.join(p, "config.json")
        with open(p, "r", encoding="utf-8") as f:
            return cls.from_dict(json.load(f))

    def needs_shapes(self) -> bool:
        return any(l["type"] == "attention" and l["mixer"].get("bias_rows") is None for l in self.layers)

    def with_shapes(self, shapes: Mapping[str, tuple]) -> "VubotarConfig":
        """The sizes that only a tensor's shape gives, from ``shapes`` (tensor name -> shape)."""
        layers = copy.deepcopy(list(self.layers))
        for i, layer in enumerate(layers):
            if layer["type"] == "attention" and layer["mixer"].get("bias_rows") is None:
                name = f"l{i}.mix.rel"
                if name not in shapes or len(shapes[name]) != 2:
                    raise ConfigError(f"the checkpoint has no matrix {name!r} to read the rows of the distance table from")
                layer["mixer"]["bias_rows"] = int(shapes[name][0])
                _check_layer(f"layers[{i}]", layer)
        return dataclasses.replace(self, layers=tuple(layers))

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"architecture": self.architecture, "vocab": self.vocab_size, "width": self.hidden_size,
                               "norm": {"eps": self.norm_eps}, "embedding": {"scale": self.embedding_scale},
                               "logit_scale": self.logit_scale, "layers": copy.deepcopy(list(self.layers))}
        if self.logit_softcap is not None:
            out["logit_softcap"] = self.logit_softcap
        if self.eos_token_id:
            out["eos_token_id"] = list(self.eos_token_id)
        return out
