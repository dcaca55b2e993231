"""The Nuzinex decoder as a ModelSpec: layers x += norm1(mixer(x)) * ls1; x += norm2(ff(x)) * ls2; x += side(x, token) (the norm
behind the sublayer, its output scaled element by element, the sublayers read the stream itself) whose mixers are, layer by
layer, windowed attention with biases, queries and keys normed over their whole projections and rotated by neighbouring
pairs (a layer may read another layer's cache); full attention with a gate beside a gated delta memory, the two added with a
weight each; or lightning attention, a memory with a constant decay per head.  Feed-forwards are W_down gelu(W_up x); every
layer ends with an input of its own by token id.  A final norm and an untied head.  Layer i's tensors start with ``l<i>.``:
norm1, norm2, ls1, ls2, mix.*, mlp.*, side.*; the rest are ``embed``, ``side.embed``, ``final.norm`` and ``head``."""

from __future__ import annotations

from typing import Any, Mapping, Optional

from ..config.nuzinex import NuzinexConfig, NuzinexLayer, window_of
from ..parts.base import LayerCall, LayerSpec, ModelSpec, PartSpec

# A small configuration for simulations and smoke runs: sizes that are all different, a layer that reads another's cache
# through a wider window, layers without feed-forward, fewer key heads than query heads, partly rotated heads, values narrower
# and wider than keys.
TINY_NUZINEX = {
    "architecture": "Nuzinex", "vocab": 93, "width": 40, "norm": {"eps": 1e-5}, "token_side": {"dim": 8}, "max_positions": 512,
    "eos_token_id": 2,
    "layers": [
        {"type": "attention",
         "mixer": {"heads": 4, "kv_heads": 2, "dim": 16, "vdim": 8, "scale": 0.3, "mask": {"size": 11}, "rot": {"base": 1000.0, "dims": 8}},
         "mlp": {"kind": "dense", "ff": 56}},
        {"type": "lightning", "mixer": {"heads": 3, "dim": 8, "vdim": 12, "decay": [0.7, 0.9, 0.99]}, "mlp": None},
        {"type": "parallel",
         "mixer": {"left": {"heads": 3, "kv_heads": 1, "dim": 12, "vdim": 16, "scale": 0.25, "rot": {"base": 300.0, "dims": 6}},
                   "right": {"heads": 4, "kv_heads": 2, "dim": 8, "vdim": 20, "conv": 3}, "left_scale": 0.7, "right_scale": 0.4},
         "mlp": {"kind": "dense", "ff": 24}},
        {"type": "attention",
         "mixer": {"heads": 6, "kv_heads": 2, "dim": 16, "vdim": 8, "scale": 0.2, "mask": {"size": 19}, "kv_from": 0,
                   "rot": {"base": 1000.0, "dims": 8}},
         "mlp": None},
    ],
}


def _attention(cfg: NuzinexConfig, m: Mapping[str, Any], layout: str, **more) -> dict:
    return dict({
        "width": cfg.width, "heads": int(m["heads"]), "kv_heads": int(m["kv_heads"]), "dim": int(m["dim"]), "vdim": int(m["vdim"]),
        "scale": float(m["scale"]), "eps": cfg.eps, "conv": 0, "qk_norm": "whole", "sink": None, "window": window_of(m),
        "position": PartSpec(layout, {"base": float(m["rot"]["base"]), "dims": int(m["rot"]["dims"]), "max_positions": cfg.max_positions}),
    }, **more)


def _mixer(cfg: NuzinexConfig, i: int, layer: NuzinexLayer, pre: str) -> PartSpec:
    m = layer.mixer
    if layer.type == "attention":
        src: Optional[int] = m.get("kv_from")
        return PartSpec("gated_attention", _attention(cfg, m, "rope_pairs", bias=True, gate=False, shared_kv=src is not None,
                                                      cache_window=cfg.cache_window(i if src is None else int(src))), pre)
    if layer.type == "lightning":
        return PartSpec("lightning", {"width": cfg.width, "heads": int(m["heads"]), "dim": int(m["dim"]), "vdim": int(m["vdim"]),
                                      "eps": cfg.eps, "decay": [float(x) for x in m["decay"]]}, pre)
    left = PartSpec("gated_attention", _attention(cfg, m["left"], "rope_halves", gate=True, shared_kv=False))
    sizes = ("heads", "kv_heads", "dim", "vdim", "conv")
    right = PartSpec("gated_delta", dict({k: int(m["right"][k]) for k in sizes}, width=cfg.width, eps=cfg.eps, unit_eps=1e-6))
    return PartSpec("side_by_side", {"width": cfg.width, "branches": [("left", left), ("right", right)],
                                     "scales": [float(m["left_scale"]), float(m["right_scale"])]}, pre)


def nuzinex_spec(cfg: NuzinexConfig) -> ModelSpec:
    layers, schedule = [], []
    for i, layer in enumerate(cfg.layers):
        pre = f"l{i}."
        norm = lambda n: PartSpec("rmsnorm", {"width": cfg.width, "eps": cfg.eps, "tensor": f"norm{n}", "gain": f"ls{n}"}, pre)
        parts = {"mixer_norm": norm(1), "mixer": _mixer(cfg, i, layer, pre + "mix."),
                 "side_input": PartSpec("token_side", {"width": cfg.width, "dim": cfg.side_dim, "offset": i * cfg.side_dim, "eps": cfg.eps},
                                        pre + "side.")}
        if layer.mlp is not None:
            parts["ffn_norm"] = norm(2)
            parts["feed_forward"] = PartSpec("mlp", {"width": cfg.width, "inter": int(layer.mlp["ff"]), "act": "gelu", "names": ("up", "down")},
                                             pre + "mlp.")
        layers.append(LayerSpec("postnorm", parts))
        src = layer.mixer.get("kv_from") if layer.type == "attention" else None
        schedule.append(LayerCall(layer=i, cache=i if src is None else int(src), writes_cache=src is None))
    return ModelSpec(
        architecture=cfg.architecture,
        vocab_size=cfg.vocab,
        width=cfg.width,
        embedding=PartSpec("embedding", {"vocab": cfg.vocab, "width": cfg.width, "tensor": "embed",
                                         "side": {"tensor": "side.embed", "width": len(cfg.layers) * cfg.side_dim}}, ""),
        layers=layers,
        schedule=schedule,
        final_norm=PartSpec("rmsnorm", {"width": cfg.width, "eps": cfg.eps, "tensor": "norm"}, "final."),
        lm_head=PartSpec("lm_head", {"vocab": cfg.vocab, "width": cfg.width, "tied": False, "tensor": "head"}, ""),
        max_positions=cfg.max_positions,
        bos_token_id=cfg.bos_token_id,
        eos_token_id=cfg.eos_token_id,
    )
