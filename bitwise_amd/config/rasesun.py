"""Typed configuration of the Rasesun decoder, read from the keys of its config.json.

Keys: ``architecture`` (the name), ``vocab``, ``width``, ``norm.eps``, ``embedding.scale``, ``logit_softcap`` (or null: the
logits are not capped), ``loop`` = {start, stop, times} or absent (layers start .. stop-1 run ``times`` times in a row), and
``layers``: a list whose entries give ``type`` (the mixer: "mamba2" or "latent_attention"), ``mixer`` (its sizes and
constants) and ``mlp`` (the feed-forward, or null for a layer without one).  Mixer keys:

* mamba2: heads, vdim, state, groups, conv (taps), norm_groups
* latent_attention: heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, rot = {base, dims}, mask = {size} (or absent: every
  earlier key is seen)

mlp: {"kind": "dense", ff} or {"kind": "moe", "expert": {ff}, "router": {experts, top}}.

Optional keys with defaults that a checkpoint's config.json need not carry: ``max_positions`` (the length of the
rotary tables and the longest request), ``bos_token_id``, ``eos_token_id``.
"""

from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Any, Dict, List, Mapping, Optional, Tuple

from .llama import ConfigError

ARCHITECTURE = "Rasesun"
MIXER_SIZES = {
    "mamba2": ("heads", "vdim", "state", "groups", "conv", "norm_groups"),
    "latent_attention": ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank"),
}
DEFAULT_MAX_POSITIONS = 1 << 16


def _positive_int(d: Any, key: str, where: str) -> int:
    v = d.get(key) if isinstance(d, Mapping) else None
    if isinstance(v, bool) or not isinstance(v, int) or v < 1:
        raise ConfigError(f"config.json: {where} needs a positive integer '{key}', got {v!r}")
    return v


def _positive(d: Any, key: str, where: str) -> float:
    v = d.get(key) if isinstance(d, Mapping) else None
    if isinstance(v, bool) or not isinstance(v, (int, float)) or not float(v) > 0:
        raise ConfigError(f"config.json: {where} needs a positive number '{key}', got {v!r}")
    return float(v)


def _check_mixer(kind: str, m: Mapping[str, Any], where: str) -> None:
    for k in MIXER_SIZES[kind]:
        _positive_int(m, k, where)
    if kind == "mamba2":
        if m["heads"] % m["groups"]:
            raise ConfigError(f"config.json: {where}: heads must be a multiple of groups")
        if (m["heads"] * m["vdim"]) % m["norm_groups"]:
            raise ConfigError(f"config.json: {where}: heads * vdim must be a multiple of norm_groups")
        return
    _positive(m, "scale", where)
    rot = m.get("rot")
    _positive(rot, "base", where + " rot")
    if _positive_int(rot, "dims", where + " rot") % 2 or rot["dims"] > m["rot_dim"]:
        raise ConfigError(f"config.json: {where}: rot.dims must be even and at most rot_dim")
    if m.get("mask") is not None:
        _positive_int(m["mask"], "size", where + " mask")


def _check_mlp(mlp: Any, where: str) -> None:
    kind = mlp.get("kind") if isinstance(mlp, Mapping) else mlp
    if kind == "dense":
        _positive_int(mlp, "ff", where + " mlp")
    elif kind == "moe":
        _positive_int(mlp.get("expert"), "ff", where + " mlp.expert")
        experts, top = (_positive_int(mlp.get("router"), k, where + " mlp.router") for k in ("experts", "top"))
        if top > experts:
            raise ConfigError(f"config.json: {where}: {top} of {experts} experts does not work out")
    else:
        raise ConfigError(f"config.json: {where} has an mlp of kind {kind!r}; known: dense, moe")


@dataclass(frozen=True)
class RasesunLayer:
    type: str
    mixer: Mapping[str, Any]
    mlp: Optional[Mapping[str, Any]]          # None: the layer has no feed-forward


@dataclass(frozen=True)
class RasesunConfig:
    architecture: str
    vocab: int
    width: int
    eps: float
    embedding_scale: float
    logit_softcap: Optional[float]            # None: the logits are not capped
    loop: Tuple[int, int, int]                # (start, stop, times); (0, 0, 1): nothing is repeated
    layers: Tuple[RasesunLayer, ...]
    max_positions: int
    bos_token_id: int
    eos_token_id: int

    @classmethod
    def from_dict(cls, d: Mapping[str, Any]) -> "RasesunConfig":
        name = d.get("architecture")
        if not isinstance(name, str):
            raise ConfigError("config.json lacks 'architecture': name")
        for key, inner in (("norm", "eps"), ("embedding", "scale")):
            if not isinstance(d.get(key), Mapping) or inner not in d[key]:
                raise ConfigError(f"config.json lacks '{key}': {{'{inner}': ...}}")
        raw_layers = d.get("layers")
        if not isinstance(raw_layers, (list, tuple)) or not raw_layers:
            raise ConfigError("config.json lacks a non-empty list 'layers'")
        layers: List[RasesunLayer] = []
        for i, entry in enumerate(raw_layers):
            where = f"layer {i}"
            kind = entry.get("type") if isinstance(entry, Mapping) else None
            if kind not in MIXER_SIZES:
                raise ConfigError(f"config.json: {where} has type {kind!r}; known: {sorted(MIXER_SIZES)}")
            mixer = entry.get("mixer")
            if not isinstance(mixer, Mapping):
                raise ConfigError(f"config.json: {where} lacks 'mixer'")
            _check_mixer(kind, mixer, f"{where} ({kind})")
            mlp = entry.get("mlp")
            if mlp is not None:
                _check_mlp(mlp, where)
            layers.append(RasesunLayer(kind, copy.deepcopy(dict(mixer)), None if mlp is None else copy.deepcopy(dict(mlp))))
        loop = d.get("loop")
        span = (0, 0, 1)
        if loop is not None:
            if not isinstance(loop, Mapping) or any(isinstance(loop.get(k), bool) or not isinstance(loop.get(k), int) for k in ("start", "stop", "times")):
                raise ConfigError("config.json: loop = {start, stop, times}, three integers")
            span = (int(loop["start"]), int(loop["stop"]), int(loop["times"]))
            if not 0 <= span[0] <= span[1] <= len(layers) or span[2] < 1:
                raise ConfigError(f"config.json: loop {dict(loop)} does not fit {len(layers)} layers")
        eos, bos = d.get("eos_token_id", -1), d.get("bos_token_id", -1)
        return cls(architecture=name, vocab=_positive_int(d, "vocab", "the model"), width=_positive_int(d, "width", "the model"),
                   eps=float(d["norm"]["eps"]), embedding_scale=float(d["embedding"]["scale"]),
                   logit_softcap=None if d.get("logit_softcap") is None else _positive(d, "logit_softcap", "the model"),
                   loop=span, layers=tuple(layers), max_positions=int(d.get("max_positions", DEFAULT_MAX_POSITIONS)),
                   bos_token_id=-1 if bos is None else int(bos), eos_token_id=-1 if eos is None else int(eos))

    def to_dict(self) -> Dict[str, Any]:
        return {
            "architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
            "embedding": {"scale": self.embedding_scale}, "logit_softcap": self.logit_softcap,
            "loop": {"start": self.loop[0], "stop": self.loop[1], "times": self.loop[2]},
            "layers": [{"type": l.type, "mixer": copy.deepcopy(dict(l.mixer)),
                        "mlp": None if l.mlp is None else copy.deepcopy(dict(l.mlp))} for l in self.layers],
            "max_positions": self.max_positions, "bos_token_id": self.bos_token_id, "eos_token_id": self.eos_token_id,
        }

    def layer_runs(self) -> List[int]:
        """The layers in the order they run."""
        start, stop, times = self.loop
        return list(range(start)) + times * list(range(start, stop)) + list(range(stop, len(self.layers)))
