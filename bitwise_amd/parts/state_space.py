"""A state-space mixer in its dual form (Mamba-2; Dao and Gu, "Transformers are SSMs: Generalized Models and Efficient
Algorithms Through Structured State Space Duality"): a matrix memory per head whose decay is a scalar per token.

    [z | x | B | C | d] = W_in h                                  inner, inner, groups * N, groups * N and heads elements
    [x | B | C]        <- silu(conv([x | B | C]))                 a causal convolution per channel, with a bias
    delta               = softplus(d + bias),  a = exp(-exp(A_log) delta)            a number a head, no clamp
    S <- a S + delta B x^T,   y = S^T C + D x                     per head, B and C shared by heads / groups neighbours
    out = W_o (norm(y silu(z)) weight)                            each of ``norm_groups`` equal parts by its own root mean square

The state of a request is the convolution's last taps - 1 inputs and S, 32-bit.  Step sizes, decays, the recurrence, gate
and norm are 32-bit in both modes, and the projections' sums enter the convolution and the step sizes unrounded.
"""

from __future__ import annotations

from typing import Dict, Optional

import torch

from ..csrc import ops
from .base import StateSpec, TensorSpec, register_mixer
from .gated_attention import max_seq_rows
from .linear import Linear
from .recurrent import _MatrixMemoryMixer


@register_mixer("mamba2")
class Mamba2(_MatrixMemoryMixer):
    """params: width, heads, vdim (value channels a head), state (N), groups, conv (taps), norm_groups, eps.
    tensors: in [2*inner + 2*groups*state + heads, width]; conv [inner + 2*groups*state, taps], conv.b; dt_bias, A_log, D
    [heads]; norm [inner]; o [width, inner], inner = heads * vdim."""

    mode = ops.RECUR_STEP_DECAY

    def __init__(self, params, runtime):
        super().__init__(dict(params, dim=int(params["state"])), runtime)
        p = params
        self.qscale = 1.0
        self.groups, self.taps, self.parts = int(p["groups"]), int(p["conv"]), int(p["norm_groups"])
        if self.heads % self.groups:
            raise ValueError(f"mamba2: {self.heads} heads do not split into {self.groups} equal groups")
        self.inner = self.heads * self.vdim
        if self.inner % self.parts:
            raise ValueError(f"mamba2: {self.inner} channels do not split into {self.parts} equal parts of the norm")
        if not 1 <= self.taps <= ops.CONV_MAX_TAPS:
            raise ValueError(f"mamba2: a convolution over {self.taps} tokens; the kernel takes 1 to {ops.CONV_MAX_TAPS}")
        gn = self.groups * self.dim
        self.channels = self.inner + 2 * gn                      # what the convolution sees: x, B, C
        self.proj_width = 2 * self.inner + 2 * gn + self.heads
        self.dt_at = self.inner + self.channels
        self.at = {"v": 0, "k": self.inner, "q": self.inner + gn}    # where x, B and C lie in a convolved row

    def tensors(self) -> Dict[str, TensorSpec]:
        return {
            "in": TensorSpec((self.proj_width, self.width)),
            "conv": TensorSpec((self.channels, self.taps), "conv"), "conv.b": TensorSpec((self.channels,), "small_bias"),
            "dt_bias": TensorSpec((self.heads,), "bias"), "A_log": TensorSpec((self.heads,), "bias"),
            "D": TensorSpec((self.heads,), "norm"),
            "norm": TensorSpec((self.inner,), "norm"),
            "o": TensorSpec((self.width, self.inner)),
        }

    def bind(self, tensors) -> None:
        dev = self.rt.device
        self.proj = Linear(tensors["in"], self.rt)
        self.o = Linear(tensors["o"], self.rt)
        put = lambda name: tensors[name].to(dev).float().contiguous()
        self.conv_w, self.conv_b = put("conv"), put("conv.b")
        self.dt_bias, self.skip, self.norm_weight = put("dt_bias"), put("D"), put("norm")
        # the decay's rate exp(A_log): in double precision, rounded once
        self.rate = tensors["A_log"].double().exp().float().to(dev).contiguous()

    def weight_bytes(self) -> int:
        small = self.conv_w.numel() + self.conv_b.numel() + 3 * self.heads + self.inner
        return self.proj.nbytes() + self.o.nbytes() + 4 * small

    def state_spec(self) -> StateSpec:
        # [taps - 1][channels] inputs of the convolution, then S [heads][state][vdim]
        return StateSpec(((self.taps - 1) * self.channels + self.heads * self.dim * self.vdim,), "float32")

    def _run(self, ctx, call, proj, target, add: bool) -> None:
        ws, rows, inner = ctx.ws, ctx.rows, self.inner
        u = ws.buffer("ssm_u", self.channels, torch.float32)
        ops.causal_conv(proj[:, inner:inner + self.channels], self.conv_w, self.conv_b, call.state, ctx.seq_rows, ctx.slots,
                        ctx.positions, ctx.nseq, max_seq_rows(ctx), u, silu=True)
        raw = ws.buffer("recur_out", inner, torch.float32)
        self._recur(ctx, call, u, proj, self.dt_at, 0, self.dt_bias, self.rate, 0.0, raw, at=self.at,
                    state=call.state[:, (self.taps - 1) * self.channels:], heads_per_key=self.heads // self.groups, skip=self.skip)
        act = ws.buffer("recur_gated", inner, self.rt.act_dtype)
        ops.gated_part_norm(raw, proj, self.norm_weight, act, ctx.positions, rows, self.parts, self.eps)
        if add:
            self.o.add_into(ws, act, target, rows)
        else:
            self.o.store(ws, act, target, rows)

    def forward(self, ctx, call, h, residual) -> None:
        self._run(ctx, call, self._project(ctx, h), residual, True)

    def forward_out(self, ctx, call, h, out) -> None:
        self._run(ctx, call, self._project(ctx, h), out, False)

    def forward_out_projected(self, ctx, call, proj, out) -> None:
        self._run(ctx, call, proj, out, False)

    def forward_between_norms(self, ctx, call, x, norm, norm_behind) -> bool:
        """Decode steps of few rows: the norm in front rides in the first product."""
        proj = ctx.ws.buffer("recur_proj", self.proj_width, torch.float32)
        if not self.proj.store_normed(x, norm, proj, ctx.rows):
            return False
        y = ctx.ws.buffer("sublayer_out", self.width, torch.float32)
        self._run(ctx, call, proj, y, False)
        norm_behind.add_normed(ctx, y, x)
        return True
