"""The Rasesun decoder as a ModelSpec: a scaled embedding; layers x += norm1b(mixer(norm1(x))); x += norm2b(ff(norm2(x)))
(a norm in front of each sublayer and one behind it) whose mixers are, layer by layer, Mamba-2's state-space memory or
windowed attention over a compressed cache whose queries go through a latent of their own and whose heads are gated; and
whose feed-forwards are xIELU units or squared-ReLU experts that a table of token ids chooses; a span of layers that runs
several times, each pass with caches and state of its own; a final norm and an untied head with soft-capped logits.
Layer i's tensors start with ``l<i>.``: norm1, norm1b, norm2, norm2b, mix.*, mlp.*; the rest are ``embed``, ``final.norm``
and ``head``."""

from __future__ import annotations

from ..config.rasesun import RasesunConfig, RasesunLayer
from ..parts.base import LayerCall, LayerSpec, ModelSpec, PartSpec

# A small configuration for simulations and smoke runs: sizes that are all different, a layer without feed-forward, the
# middle layers run three times, two experts a token, one group and several, the norm in one part and in several.
TINY_RASESUN = {
    "architecture": "Rasesun", "vocab": 97, "width": 40, "norm": {"eps": 1e-5}, "embedding": {"scale": 2.5}, "logit_softcap": 12.0,
    "max_positions": 512, "eos_token_id": 2, "loop": {"start": 1, "stop": 3, "times": 3},
    "layers": [
        {"type": "mamba2", "mixer": {"heads": 4, "vdim": 12, "state": 8, "groups": 2, "conv": 3, "norm_groups": 3},
         "mlp": {"kind": "moe", "expert": {"ff": 24}, "router": {"experts": 6, "top": 2}}},
        {"type": "latent_attention",
         "mixer": {"heads": 3, "dim": 8, "rot_dim": 4, "vdim": 12, "q_rank": 16, "kv_rank": 20, "scale": 0.3, "mask": {"size": 21},
                   "rot": {"base": 1000.0, "dims": 4}},
         "mlp": {"kind": "dense", "ff": 56}},
        {"type": "mamba2", "mixer": {"heads": 3, "vdim": 16, "state": 20, "groups": 1, "conv": 4, "norm_groups": 1}, "mlp": None},
        {"type": "latent_attention",
         "mixer": {"heads": 5, "dim": 12, "rot_dim": 8, "vdim": 8, "q_rank": 24, "kv_rank": 16, "scale": 0.25, "mask": {"size": 9},
                   "rot": {"base": 300.0, "dims": 8}},
         "mlp": {"kind": "moe", "expert": {"ff": 16}, "router": {"experts": 5, "top": 3}}},
    ],
}


def _mixer(cfg: RasesunConfig, layer: RasesunLayer, pre: str) -> PartSpec:
    m = layer.mixer
    if layer.type == "mamba2":
        sizes = ("heads", "vdim", "state", "groups", "conv", "norm_groups")
        return PartSpec("mamba2", dict({k: int(m[k]) for k in sizes}, width=cfg.width, eps=cfg.eps), pre)
    sizes = ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank")
    return PartSpec("latent_attention", dict(
        {k: int(m[k]) for k in sizes}, width=cfg.width, eps=cfg.eps, scale=float(m["scale"]),
        window=None if m.get("mask") is None else int(m["mask"]["size"]), sink=False, gate=True,
        position=PartSpec("rope_pairs", {"base": float(m["rot"]["base"]), "dims": int(m["rot"]["dims"]),
                                         "max_positions": cfg.max_positions})), pre)


def _feed_forward(cfg: RasesunConfig, layer: RasesunLayer, pre: str) -> PartSpec:
    mlp = layer.mlp
    if mlp["kind"] == "dense":
        return PartSpec("mlp", {"width": cfg.width, "inter": int(mlp["ff"]), "act": "xielu"}, pre)
    ro = mlp["router"]
    return PartSpec("moe", {"width": cfg.width, "experts": int(ro["experts"]), "top": int(ro["top"]), "ff": int(mlp["expert"]["ff"]),
                            "table": cfg.vocab, "form": "plain"}, pre)


def rasesun_spec(cfg: RasesunConfig) -> ModelSpec:
    layers = []
    for i, layer in enumerate(cfg.layers):
        pre = f"l{i}."
        norm = lambda tensor: PartSpec("rmsnorm", {"width": cfg.width, "eps": cfg.eps, "tensor": tensor}, pre)
        parts = {"mixer_norm": norm("norm1"), "mixer": _mixer(cfg, layer, pre + "mix."), "mixer_post_norm": norm("norm1b")}
        if layer.mlp is not None:
            parts.update(ffn_norm=norm("norm2"), ffn_post_norm=norm("norm2b"), feed_forward=_feed_forward(cfg, layer, pre + "mlp."))
        layers.append(LayerSpec("sandwich", parts))
    head = {"vocab": cfg.vocab, "width": cfg.width, "tied": False, "tensor": "head"}
    return ModelSpec(
        architecture=cfg.architecture,
        vocab_size=cfg.vocab,
        width=cfg.width,
        embedding=PartSpec("embedding_sum", {"vocab": cfg.vocab, "width": cfg.width, "tensor": "embed", "scale": cfg.embedding_scale}, ""),
        layers=layers,
        # every run of a layer has a cache and state of its own
        schedule=[LayerCall(layer=i, cache=n) for n, i in enumerate(cfg.layer_runs())],
        final_norm=PartSpec("rmsnorm", {"width": cfg.width, "eps": cfg.eps, "tensor": "norm"}, "final."),
        lm_head=PartSpec("lm_head", head, "") if cfg.logit_softcap is None else PartSpec("lm_head_softcap", dict(head, cap=cfg.logit_softcap), ""),
        max_positions=cfg.max_positions,
        bos_token_id=cfg.bos_token_id,
        eos_token_id=cfg.eos_token_id,
    )
