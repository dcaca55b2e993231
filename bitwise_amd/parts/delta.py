"""A matrix memory per head written by the gated delta rule (Yang, Kautz and Hatamizadeh, "Gated Delta Networks: Improving
Mamba2 with Delta Rule"): what a key reads from the decayed memory is replaced towards the value by a step size.

    q, k, v = silu(conv(W_q h)), silu(conv(W_k h)), silu(conv(W_v h))     a causal convolution over `taps` tokens per channel
    q, k    = unit(q) dim^(-1/2), unit(k)                                 x / sqrt(sum x^2 + 1e-6) per head
    b = sigmoid(W_b h),  a = exp(-exp(A_log) softplus(W_a h + dt_bias))   a number a head
    S <- a S;  S <- S + k (b (v - S^T k))^T;  o = S^T q                   per head; heads / kv_heads neighbours share q and k
    out = W_o (o / sqrt(mean(o^2) + eps) * weight * silu(W_g h))          the norm per head, one weight for all heads

The state of a request is S and the convolution's last taps - 1 inputs, 32-bit.  Step sizes, decays, unit norms, the recurrence,
norm and gate are 32-bit in both modes, and the projections' sums enter the convolution and the gates unrounded.
"""

from __future__ import annotations

from typing import Dict

import torch

from ..csrc import ops
from .base import StateSpec, TensorSpec, register_mixer
from .gated_attention import max_seq_rows
from .linear import Linear
from .recurrent import _MatrixMemoryMixer


@register_mixer("gated_delta")
class GatedDelta(_MatrixMemoryMixer):
    """params: width, heads, kv_heads (of the queries and keys), dim, vdim, conv (taps), eps; optional unit_eps (1e-6).
    tensors: q, k [kv_heads*dim, width]; v, g [heads*vdim, width]; b, a [heads, width]; q.conv, k.conv, v.conv [channels, taps];
    A_log, dt_bias [heads]; norm [vdim]; o [width, heads*vdim]."""

    mode = ops.RECUR_DELTA
    gate_kind = ops.GATE_SILU
    per_head_norm_weight = False
    passes = False

    def __init__(self, params, runtime):
        super().__init__(params, runtime)
        p = params
        self.qscale = 1.0                     # (the queries arrive scaled)
        self.kv_heads, self.taps = int(p["kv_heads"]), int(p["conv"])
        self.unit_eps = float(p.get("unit_eps", 1e-6))
        if self.heads % self.kv_heads:
            raise ValueError(f"gated_delta: {self.heads} heads do not share {self.kv_heads} key heads evenly")
        if not 1 <= self.taps <= ops.CONV_MAX_TAPS:
            raise ValueError(f"gated_delta: a convolution over {self.taps} tokens; the kernel takes 1 to {ops.CONV_MAX_TAPS}")
        qk = self.kv_heads * self.dim
        self.channels = 2 * qk + self.heads * self.vdim           # what the convolution sees: q, k, v
        self.at = {"q": 0, "k": qk, "v": 2 * qk}                  # where they lie in a convolved row
        self.memory = self.heads * self.dim * self.vdim
        self.conv_w = self.dt_bias = self.rate = None

    def _stack_sizes(self):
        qk, hv = self.kv_heads * self.dim, self.heads * self.vdim
        return [("q", qk), ("k", qk), ("v", hv), ("g", hv), ("b", self.heads), ("a", self.heads)]

    def tensors(self) -> Dict[str, TensorSpec]:
        out = super().tensors()
        for name, n in (("q", self.kv_heads * self.dim), ("k", self.kv_heads * self.dim), ("v", self.heads * self.vdim)):
            out[name + ".conv"] = TensorSpec((n, self.taps), "conv")
        out["A_log"] = TensorSpec((self.heads,), "bias")
        out["dt_bias"] = TensorSpec((self.heads,), "bias")
        return out

    def bind(self, tensors) -> None:
        dev = self.rt.device
        self._bind_common(tensors)
        self.conv_w = torch.cat([tensors[n + ".conv"].to(dev).float() for n in ("q", "k", "v")], dim=0).contiguous()
        self.dt_bias = tensors["dt_bias"].to(dev).float().contiguous()
        # the decay's rate exp(A_log): in double precision, rounded once
        self.rate = tensors["A_log"].double().exp().float().to(dev).contiguous()

    def weight_bytes(self) -> int:
        return self.proj.nbytes() + self.o.nbytes() + 4 * (self.conv_w.numel() + 2 * self.heads + self.vdim)

    def state_spec(self) -> StateSpec:
        # S [heads][vdim][dim], then [taps - 1][channels] inputs of the convolution
        return StateSpec((self.memory + (self.taps - 1) * self.channels,), "float32")

    def _run(self, ctx, call, y, target, add: bool) -> None:
        ws = ctx.ws
        u = ws.buffer("delta_u", self.channels, torch.float32)
        gates = ws.buffer("delta_gates", 2 * self.heads + self.kv_heads, torch.float32)
        ops.conv_heads(y, self.conv_w, call.state[:, self.memory:] if self.taps > 1 else None, y, self.offsets["a"], self.offsets["b"],
                       self.dt_bias, self.rate, self.kv_heads, self.dim, ctx.seq_rows, ctx.slots, ctx.positions, ctx.nseq,
                       max_seq_rows(ctx), u, gates, float(self.dim) ** -0.5, self.unit_eps)
        raw = ws.buffer("recur_out", self.heads * self.vdim, torch.float32)
        self._recur(ctx, call, u, gates, 0, self.heads, None, None, 0.0, raw, at=self.at, heads_per_key=self.heads // self.kv_heads)
        self._finish(ctx, y, raw, target, add)

    def forward(self, ctx, call, h, residual) -> None:
        self._run(ctx, call, self._project(ctx, h), residual, True)

    def forward_out(self, ctx, call, h, out) -> None:
        self._run(ctx, call, self._project(ctx, h), out, False)

    def forward_out_projected(self, ctx, call, proj, out) -> None:
        self._run(ctx, call, proj, out, False)
