"""Typed configuration of the Taluvik decoder: layers of three kinds of mixers whose two branches run side by side,
layers that run on another layer's weights.

``config.json`` gives: ``architecture`` "Taluvik", ``vocab``, ``width``, ``norm.eps``, ``embedding.scale``,
``residual_mult`` and ``layers``, one entry per layer run: ``type`` and ``mixer``,

* "delta": {heads, kv_heads, dim, vdim, conv};
* "mamba1": {inner, state, dt_rank, conv};
* "attention": {heads, kv_heads, dim, vdim, scale, rot {dims, base, scaling {factor, low, high, original}?}?, softcap?,
  mask {size}?};

``mlp`` = {kind "dense", ff} or null, and optionally ``weights_of``: the layer whose tensors this one runs on (its other
keys are then that layer's).
"""
from __future__ import annotations

import copy
import json
import os
from dataclasses import dataclass, field
from typing import Any, Mapping

from tensorline_amd.config.model_config import ConfigError

LAYER_TYPES = ("delta", "mamba1", "attention")
_INT_KEYS = {"delta": ("heads", "kv_heads", "dim", "vdim", "conv"),
             "mamba1": ("inner", "state", "dt_rank", "conv"),
             "attention": ("heads", "kv_heads", "dim", "vdim")}


def _positive_int(where: str, d: Any, key: str) -> int:
    v = d.get(key) if isinstance(d, Mapping) else None
    if isinstance(v, bool) or not isinstance(v, int) or v <= 0:
        raise ConfigError(f"config.json: {where}.{key} must be a positive integer, got {v!r}")
    return v


def _number(where: str, d: Any, key: str) -> float:
    v = d.get(key) if isinstance(d, Mapping) else None
    if isinstance(v, bool) or not isinstance(v, (int, float)):
        raise ConfigError(f"config.json: {where}.{key} must be a number, got {v!r}")
    return float(v)


def _check_rot(where: str, rot: Any, dim: int) -> None:
    if not isinstance(rot, Mapping):
        raise ConfigError(f"config.json: {where} must be an object")
    dims = _positive_int(where, rot, "dims")
    if dims % 2 or dims > dim:
        raise ConfigError(f"config.json: {where}.dims {dims} must be even and at most {dim}")
    if not _number(where, rot, "base") > 0.0:
        raise ConfigError(f"config.json: {where}.base must be positive")
    sc = rot.get("scaling")
    if sc is not None:
        factor, low, high, original = (_number(where + ".scaling", sc, k) for k in ("factor", "low", "high", "original"))
        if min(factor, low, original) <= 0.0 or high < low:
            raise ConfigError(f"config.json: {where}.scaling: factor, low and original must be positive and high at least low")


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
    if "heads" in _INT_KEYS[kind] and mixer["heads"] % mixer["kv_heads"]:
        raise ConfigError(f"config.json: {where_m}: {mixer['heads']} heads are not a multiple of {mixer['kv_heads']} kv_heads")
    if kind == "attention":
        if not _number(where_m, mixer, "scale") > 0.0:
            raise ConfigError(f"config.json: {where_m}.scale must be positive")
        if mixer.get("softcap") is not None and not _number(where_m, mixer, "softcap") > 0.0:
            raise ConfigError(f"config.json: {where_m}.softcap must be positive")
        if mixer.get("mask") is not None:
            _positive_int(where_m + ".mask", mixer["mask"], "size")
        if mixer.get("rot") is not None:
            _check_rot(where_m + ".rot", mixer["rot"], mixer["dim"])
    mlp = layer.get("mlp")
    if mlp is not None:
        if not isinstance(mlp, Mapping) or mlp.get("kind") != "dense":
            raise ConfigError(f"config.json: {where}.mlp.kind {mlp.get('kind') if isinstance(mlp, Mapping) else mlp!r} is unknown; known: dense")
        _positive_int(where + ".mlp", mlp, "ff")


@dataclass(frozen=True)
class TaluvikConfig:
    vocab_size: int
    hidden_size: int
    layers: tuple = ()                      # the entries of config.json's ``layers``, checked
    norm_eps: float = 1e-6
    embedding_scale: float = 1.0
    residual_mult: float = 1.0
    eos_token_id: tuple[int, ...] = ()
    max_position_embeddings: int = 1 << 30
    architecture: str = "Taluvik"
    extra: Mapping[str, Any] = field(default_factory=dict, compare=False, hash=False)

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    def weight_layer(self, i: int) -> int:
        """The layer whose tensors layer ``i`` runs on (itself, unless ``weights_of`` names another)."""
        seen = {i}
        while self.layers[i].get("weights_of") is not None:
            i = self.layers[i]["weights_of"]
            if i in seen:
                raise ConfigError(f"config.json: layers[{i}].weights_of leads back to itself")
            seen.add(i)
        return i

    @classmethod
    def from_dict(cls, d: Mapping[str, Any]) -> "TaluvikConfig":
        vocab, width = _positive_int("", d, "vocab"), _positive_int("", d, "width")
        raw_layers = d.get("layers")
        if not isinstance(raw_layers, list) or not raw_layers:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        eps = _number("norm", d.get("norm"), "eps")
        layers = []
        for i, layer in enumerate(raw_layers):
            _check_layer(f"layers[{i}]", layer)
            of = layer.get("weights_of")
            if of is not None and (isinstance(of, bool) or not isinstance(of, int) or not 0 <= of < len(raw_layers) or of == i):
                raise ConfigError(f"config.json: layers[{i}].weights_of {of!r} must name another layer")
            layers.append(copy.deepcopy(dict(layer)))
        eos = d.get("eos_token_id")
        eos_ids = () if eos is None else tuple(int(e) for e in eos) if isinstance(eos, (list, tuple)) else (int(eos),)
        known = {"architecture", "architectures", "vocab", "width", "layers", "norm", "embedding", "residual_mult", "eos_token_id",
                 "max_position_embeddings"}
        embedding = d.get("embedding") or {}
        out = cls(vocab_size=vocab, hidden_size=width, layers=tuple(layers), norm_eps=eps,
                  embedding_scale=float(embedding.get("scale", 1.0)), residual_mult=float(d.get("residual_mult", 1.0)),
                  eos_token_id=eos_ids, max_position_embeddings=int(d.get("max_position_embeddings", 1 << 30)),
                  extra={k: v for k, v in d.items() if k not in known})
        for i, layer in enumerate(layers):
            j = out.weight_layer(i)
            for key in ("type", "mixer", "mlp"):
                if layer.get(key) != layers[j].get(key):
                    raise ConfigError(f"config.json: layers[{i}] runs on the weights of layers[{j}], but its {key} differs")
        return out

    @classmethod
    def from_json(cls, path: str | os.PathLike) -> "TaluvikConfig":
        p = os.fspath(path)
        if os.path.isdir(p):
            p = os.path.join(p, "config.json")
        with open(p, "r", encoding="utf-8") as f:
            return cls.from_dict(json.load(f))

    def to_dict(self) -> dict[str, Any]:
        out: dict[str, Any] = {"architecture": self.architecture, "vocab": self.vocab_size, "width": self.hidden_size,
                               "norm": {"eps": self.norm_eps}, "embedding": {"scale": self.embedding_scale},
                               "residual_mult": self.residual_mult, "layers": copy.deepcopy(list(self.layers))}
        if self.eos_token_id:
            out["eos_token_id"] = list(self.eos_token_id)
        return out
