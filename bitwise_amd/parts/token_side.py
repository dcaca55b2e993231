"""A per-layer input by token id: every layer has its own columns of one table with a row per token, and what it reads there,
gated by the stream, is added to the stream behind the layer's sublayers.

    e = table[token, offset : offset + dim]
    g = gelu_tanh(W_gate x) * e
    x <- x + norm(W_proj g),        norm(y) = y / sqrt(mean(y^2) + eps) * weight

The table belongs to the embedding part (``side``), which leaves it in the pass's notes.
"""

from __future__ import annotations

from typing import Dict, Optional

import torch

from ..csrc import ops
from .base import SideInput, TensorSpec, register_side_input
from .linear import Linear


@register_side_input("token_side")
class TokenSide(SideInput):
    """params: width, dim, offset (of the layer's columns in the table), eps.  tensors: gate [dim, width]; proj [width, dim];
    norm [width].  The table's row, the activation and the norm are 32-bit in both modes; bfloat16 mode rounds what the two
    products read."""

    graph_safe = True
    launches_through_ops = True

    def __init__(self, params, runtime):
        super().__init__(params, runtime)
        self.width, self.dim, self.offset = int(params["width"]), int(params["dim"]), int(params["offset"])
        self.eps = float(params["eps"])
        self.gate: Optional[Linear] = None
        self.proj: Optional[Linear] = None
        self.norm_weight: Optional[torch.Tensor] = None

    def tensors(self) -> Dict[str, TensorSpec]:
        return {"gate": TensorSpec((self.dim, self.width)), "proj": TensorSpec((self.width, self.dim)),
                "norm": TensorSpec((self.width,), "norm")}

    def bind(self, tensors) -> None:
        self.gate, self.proj = Linear(tensors["gate"], self.rt), Linear(tensors["proj"], self.rt)
        self.norm_weight = tensors["norm"].to(self.rt.device).float().contiguous()

    def weight_bytes(self) -> int:
        return self.gate.nbytes() + self.proj.nbytes() + 4 * self.width

    def forward_add(self, ctx, h, x, rounded=None) -> None:
        ws, rows = ctx.ws, ctx.rows
        table = ctx.forward_notes.get("token_side_table")
        if table is None or table.shape[1] < self.offset + self.dim:
            raise ValueError("token_side: the embedding holds no side table with this layer's columns")
        e, feedback = table[:, self.offset:self.offset + self.dim], getattr(ctx, "token_feedback", None)
        g = ws.buffer("side_gated", self.dim, self.rt.act_dtype)
        if self.gate.mfma and h.dtype == torch.bfloat16 and ops.side_gemm_ok(rows, self.gate.weight, e):
            ops.gemm_side_bf16(h, self.gate.weight, ctx.tokens, feedback, e, g, rows)      # (decode steps: one launch, the same bits)
        else:
            z = ws.buffer("side_gate", self.dim, torch.float32)
            self.gate.store(ws, h, z, rows)
            ops.side_gate(z, ctx.tokens, feedback, e, g, rows)
        y = ws.buffer("side_out", self.width, torch.float32)
        self.proj.store(ws, g, y, rows)
        ops.norm_add(y, self.norm_weight, x, rows, self.eps, rounded)
