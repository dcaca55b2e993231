"""Typed configuration of the Nuzinex decoder, read from the keys of its config.json.

Keys: ``architecture`` (the name), ``vocab``, ``width``, ``norm.eps``, ``token_side.dim`` (a layer's columns in the side table of
token rows), and ``layers``: a list whose entries give ``type`` (the mixer: "attention", "parallel" or "lightning"), ``mixer``
(its sizes and constants) and ``mlp`` (the feed-forward, or null for a layer without one).  Mixer keys:

* attention: heads, kv_heads, dim, vdim, scale, rot = {base, dims}; mask = {size} (the window; absent: every earlier key);
  optional kv_from (the layer whose cached keys and values this layer reads instead of making its own)
* parallel: left = {heads, kv_heads, dim, vdim, scale, rot, mask or absent}, right = {heads, kv_heads, dim, vdim, conv},
  left_scale, right_scale
* lightning: heads, dim, vdim, decay (a number per head)

mlp: {"kind": "dense", "ff"}.

Optional keys with defaults that a checkpoint's config.json need not carry: ``max_positions`` (the length of the
rotary tables and the longest request), ``bos_token_id``, ``eos_token_id``.
"""

from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Any, Dict, List, Mapping, Optional, Tuple

from .llama import ConfigError

ARCHITECTURE = "Nuzinex"
ATTENTION_SIZES = ("heads", "kv_heads", "dim", "vdim")
DELTA_SIZES = ("heads", "kv_heads", "dim", "vdim", "conv")
LIGHTNING_SIZES = ("heads", "dim", "vdim")
TYPES = ("attention", "lightning", "parallel")
DEFAULT_MAX_POSITIONS = 1 << 16


def _positive_int(d: Mapping[str, Any], key: str, where: str) -> int:
    v = d.get(key)
    if isinstance(v, bool) or not isinstance(v, int) or v < 1:
        raise ConfigError(f"config.json: {where} needs a positive integer '{key}', got {v!r}")
    return v


def _number(d: Mapping[str, Any], key: str, where: str) -> float:
    v = d.get(key)
    if isinstance(v, bool) or not isinstance(v, (int, float)):
        raise ConfigError(f"config.json: {where} needs a number '{key}', got {v!r}")
    return float(v)


def window_of(mixer: Mapping[str, Any]) -> Optional[int]:
    """The window of an attention mixer, or None."""
    return None if mixer.get("mask") is None else int(mixer["mask"]["size"])


def _heads(m: Mapping[str, Any], sizes: Tuple[str, ...], where: str) -> None:
    for k in sizes:
        _positive_int(m, k, where)
    if "kv_heads" in sizes and m["heads"] % m["kv_heads"]:
        raise ConfigError(f"config.json: {where}: heads must be a multiple of kv_heads")


def _check_attention(m: Mapping[str, Any], where: str) -> None:
    _heads(m, ATTENTION_SIZES, where)
    if not _number(m, "scale", where) > 0:
        raise ConfigError(f"config.json: {where}: scale must be positive")
    rot = m.get("rot")
    if not isinstance(rot, Mapping) or "base" not in rot or "dims" not in rot:
        raise ConfigError(f"config.json: {where} needs rot = {{base, dims}}")
    if isinstance(rot["dims"], bool) or not isinstance(rot["dims"], int) or rot["dims"] % 2 or not 0 <= rot["dims"] <= m["dim"]:
        raise ConfigError(f"config.json: {where}: rot.dims must be even and at most dim")
    if not float(rot["base"]) > 0.0:
        raise ConfigError(f"config.json: {where}: rot.base must be positive")
    mask = m.get("mask")
    if mask is not None:
        if not isinstance(mask, Mapping):
            raise ConfigError(f"config.json: {where}: mask = {{size}}")
        _positive_int(mask, "size", where + " mask")


@dataclass(frozen=True)
class NuzinexLayer:
    type: str
    mixer: Mapping[str, Any]
    mlp: Optional[Mapping[str, Any]]          # None: the layer has no feed-forward


@dataclass(frozen=True)
class NuzinexConfig:
    architecture: str
    vocab: int
    width: int
    eps: float
    side_dim: int
    layers: Tuple[NuzinexLayer, ...]
    max_positions: int
    bos_token_id: int
    eos_token_id: int

    @classmethod
    def from_dict(cls, d: Mapping[str, Any]) -> "NuzinexConfig":
        name = d.get("architecture")
        if not isinstance(name, str):
            raise ConfigError("config.json lacks 'architecture': name")
        norm, side = d.get("norm"), d.get("token_side")
        if not isinstance(norm, Mapping) or "eps" not in norm:
            raise ConfigError("config.json lacks 'norm': {'eps': ...}")
        if not isinstance(side, Mapping):
            raise ConfigError("config.json lacks 'token_side': {'dim': ...}")
        raw_layers = d.get("layers")
        if not isinstance(raw_layers, (list, tuple)) or not raw_layers:
            raise ConfigError("config.json lacks a non-empty list 'layers'")
        layers: List[NuzinexLayer] = []
        for i, entry in enumerate(raw_layers):
            where = f"layer {i}"
            kind = entry.get("type") if isinstance(entry, Mapping) else None
            if kind not in TYPES:
                raise ConfigError(f"config.json: {where} has type {kind!r}; known: {list(TYPES)}")
            m = entry.get("mixer")
            if not isinstance(m, Mapping):
                raise ConfigError(f"config.json: {where} lacks 'mixer'")
            if kind == "attention":
                _check_attention(m, where)
                src = m.get("kv_from")
                if src is not None:
                    ok = isinstance(src, int) and not isinstance(src, bool) and 0 <= src < i and layers[src].type == "attention" \
                        and layers[src].mixer.get("kv_from") is None
                    if not ok:
                        raise ConfigError(f"config.json: {where}: kv_from must name an earlier attention layer with keys and values of its own")
                    other = layers[src].mixer
                    if any(other[k] != m[k] for k in ("kv_heads", "dim", "vdim")):
                        raise ConfigError(f"config.json: {where}: kv_from names a layer with other key/value heads")
            elif kind == "parallel":
                left, right = m.get("left"), m.get("right")
                if not isinstance(left, Mapping) or not isinstance(right, Mapping):
                    raise ConfigError(f"config.json: {where} needs mixer.left and mixer.right")
                _check_attention(left, where + " left")
                _heads(right, DELTA_SIZES, where + " right")
                for k in ("left_scale", "right_scale"):
                    _number(m, k, where)
            else:
                _heads(m, LIGHTNING_SIZES, where)
                decay = m.get("decay")
                if not isinstance(decay, (list, tuple)) or len(decay) != m["heads"] or any(
                        isinstance(x, bool) or not isinstance(x, (int, float)) or not 0.0 <= float(x) <= 1.0 for x in decay):
                    raise ConfigError(f"config.json: {where}: decay must give a number in [0, 1] per head")
            mlp = entry.get("mlp")
            if mlp is not None:
                if not isinstance(mlp, Mapping) or mlp.get("kind") != "dense":
                    raise ConfigError(f"config.json: {where} has an mlp of kind {mlp.get('kind') if isinstance(mlp, Mapping) else mlp!r}; known: dense")
                _positive_int(mlp, "ff", where + " mlp")
            layers.append(NuzinexLayer(kind, copy.deepcopy(dict(m)), None if mlp is None else copy.deepcopy(dict(mlp))))
        eos, bos = d.get("eos_token_id", -1), d.get("bos_token_id", -1)
        return cls(architecture=name, vocab=_positive_int(d, "vocab", "the model"), width=_positive_int(d, "width", "the model"),
                   eps=_number(norm, "eps", "norm"), side_dim=_positive_int(side, "dim", "token_side"), layers=tuple(layers),
                   max_positions=int(d.get("max_positions", DEFAULT_MAX_POSITIONS)),
                   bos_token_id=-1 if bos is None else int(bos), eos_token_id=-1 if eos is None else int(eos))

    def to_dict(self) -> Dict[str, Any]:
        return {
            "architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
            "token_side": {"dim": self.side_dim},
            "layers": [{"type": l.type, "mixer": copy.deepcopy(dict(l.mixer)),
                        "mlp": None if l.mlp is None else copy.deepcopy(dict(l.mlp))} for l in self.layers],
            "max_positions": self.max_positions, "bos_token_id": self.bos_token_id, "eos_token_id": self.eos_token_id,
        }

    def cache_window(self, i: int) -> Optional[int]:
        """How far back the keys of attention layer i are read, by the layer itself and by those that read its cache (None:
        as far as the request goes)."""
        readers = [l.mixer for n, l in enumerate(self.layers) if l.type == "attention" and (n == i or l.mixer.get("kv_from") == i)]
        windows = [window_of(m) for m in readers]
        return None if None in windows else max(windows)
