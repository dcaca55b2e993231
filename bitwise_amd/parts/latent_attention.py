"""Causal attention over a compressed cache: per token one latent vector (RMS-normed) and one rotated key
part shared by all heads are cached; a head's key is [W_uk c | rotated part], its value W_uv c.

The scores are taken in the cache's own space: q_unrotated . (W_uk c) = (W_uk^T q_unrotated) . c, so a head's
query becomes [W_uk^T q_unrotated | q_rotated] and one dot product with the cached vector is the score; the
softmax-weighted sum of cached latents is projected to the head's values by W_uv afterwards.  The softmax may have
a sink: one learned number per head that enters the denominator as exp(sink) beside the keys' terms (nothing is
looked up for it, nothing is added to the output for it, and the score scale does not apply to it).  The queries may go
through an RMS-normed latent of their own, and a head's output may be multiplied by a sigmoid gate of the input.

Rotations, the latent's norm, scores and softmax weights are 32-bit in both modes; the cache holds the mode's
activation dtype.
"""

from __future__ import annotations

from typing import Dict, Optional

import numpy as np
import torch

from ..csrc import ops
from .base import CacheSpec, Mixer, TensorSpec, lookup, register_mixer, POSITION_ENCODINGS
from .linear import Linear

ROWS_PER_PROMPT_TILE = 4        # the 32-bit kernel: 16 query vectors a workgroup, 4 rows x 4 heads or a single token's 16 heads


def _tiles(ctx, rows_per_tile: int):
    """(prompt tiles, count, single-token tiles, count): tiles (first row, rows, request, 0) of up to ``rows_per_tile``
    consecutive rows of a request; single tokens apart (their workgroups take 16 heads each).  None with a positive
    count: tile t is row t of request t (a step of one row per request)."""
    if getattr(ctx, "one_row_per_request", False):
        return None, 0, None, ctx.rows

    def make():
        many, single = [], []
        for i, s in enumerate(ctx.segments):
            n, r0 = len(s.tokens), ctx.seq_start[i]
            if n == 1:
                single.append((r0, 1, i, 0))
                continue
            for off in range(0, n, rows_per_tile):
                many.append((r0 + off, min(rows_per_tile, n - off), i, 0))
        both = torch.from_numpy(np.asarray(many + single, np.int32).reshape(-1, 4)).to(ctx.device)
        return (both[:len(many)].contiguous() if many else None, len(many),
                both[len(many):].contiguous() if single else None, len(single))

    return ctx.memo(("shared_key_tiles", rows_per_tile), make)


@register_mixer("latent_attention")
class LatentAttention(Mixer):
    """params: width, heads, dim (unrotated query/key elements a head), rot_dim (rotated ones), vdim, kv_rank, scale, eps
    (of the latent's norm), window (None: all keys), position (PartSpec of the rotary tables; it may rotate fewer than
    rot_dim elements, the rest of the rotated part passes unchanged; its pairs are neighbours if its ``layout`` says
    "pairs", else half the rotated elements apart), q_rank (None: the queries are projected from the input), sink (True),
    gate (False; True: one logit a head).
    tensors: q [heads*(dim+rot_dim), width], or with q_rank dq [q_rank, width], dq.norm [q_rank] and uq
    [heads*(dim+rot_dim), q_rank]; dkv [kv_rank+rot_dim, width]; dkv.norm [kv_rank]; uk [heads*dim, kv_rank];
    uv [heads*vdim, kv_rank]; with sink: sink [heads]; with gate: g [heads, width]; o [width, heads*vdim]."""

    launches_through_ops = True

    def __init__(self, params, runtime):
        super().__init__(params, runtime)
        p = params
        self.width, self.heads = int(p["width"]), int(p["heads"])
        self.dim, self.rot, self.vdim, self.rank = int(p["dim"]), int(p["rot_dim"]), int(p["vdim"]), int(p["kv_rank"])
        self.scale, self.eps = float(p["scale"]), float(p["eps"])
        self.window: Optional[int] = p.get("window")
        self.q_rank = int(p.get("q_rank") or 0)
        self.has_sink, self.has_gate = bool(p.get("sink", True)), bool(p.get("gate", False))
        self.key_width = self.rank + self.rot
        if self.rank > 512:
            raise ValueError(f"latent_attention: a latent of {self.rank} elements; the kernel takes up to 512")
        pos = p["position"]
        self.position = lookup(POSITION_ENCODINGS, "position encoding", pos.kind).shared(pos.params, runtime)
        self.rotary = int(getattr(self.position, "rotary_dim", 0))
        if self.rotary % 2 or self.rotary > self.rot:
            raise ValueError(f"latent_attention: the position encoding rotates {self.rotary} elements, the rotated part has {self.rot}")
        self.pairs = getattr(self.position, "layout", "halves") == "pairs"
        self.graph_safe = bool(getattr(self.position, "graph_safe", False))
        self.cos = self.sin = None
        self.proj: Optional[Linear] = None
        self.uq: Optional[Linear] = None
        self.o: Optional[Linear] = None
        self.sink: Optional[torch.Tensor] = None
        self.q_norm: Optional[torch.Tensor] = None
        # bfloat16 mode: the attention runs on the matrix cores and keeps the latents a second time, transposed within
        # their pages, as the values (the page sizes it takes: powers of two from 8 on); the 32-bit mode reads values and keys
        # from the one copy
        self.on_matrix_cores = bool(runtime.bf16) and self.key_width % 8 == 0
        # heads that share a wave's 16 query vectors in prompt portions: the power of two from the number of heads up
        self.heads_per_group = 1
        while self.heads_per_group < min(self.heads, 16):
            self.heads_per_group *= 2

    def tensors(self) -> Dict[str, TensorSpec]:
        nq = self.heads * (self.dim + self.rot)
        out = {}
        if self.q_rank:
            out["dq"] = TensorSpec((self.q_rank, self.width))
            out["dq.norm"] = TensorSpec((self.q_rank,), "norm")
            out["uq"] = TensorSpec((nq, self.q_rank))
        else:
            out["q"] = TensorSpec((nq, self.width))
        out["dkv"] = TensorSpec((self.key_width, self.width))
        out["dkv.norm"] = TensorSpec((self.rank,), "norm")
        out["uk"] = TensorSpec((self.heads * self.dim, self.rank))
        out["uv"] = TensorSpec((self.heads * self.vdim, self.rank))
        if self.has_sink:
            out["sink"] = TensorSpec((self.heads,), "bias")
        if self.has_gate:
            out["g"] = TensorSpec((self.heads, self.width))
        out["o"] = TensorSpec((self.width, self.heads * self.vdim))
        return out

    def bind(self, tensors) -> None:
        self.cos, self.sin = self.position.tables()
        # everything that reads the mixer's input is one product: [queries or their latent | down projection | gate]
        stack = [tensors["dq" if self.q_rank else "q"], tensors["dkv"]] + ([tensors["g"]] if self.has_gate else [])
        if len({t.dtype for t in stack}) != 1:
            raise ValueError("the projections of the mixer's input must be stored in one dtype to be stacked")
        self.q_off, self.dkv_off = 0, stack[0].shape[0]
        self.gate_off = self.dkv_off + self.key_width
        self.proj = Linear(torch.cat(stack, dim=0), self.rt)
        if self.q_rank:
            self.uq = Linear(tensors["uq"], self.rt)
            self.q_norm = tensors["dq.norm"].to(self.rt.device).float().contiguous()
        self.o = Linear(tensors["o"], self.rt)
        dev = self.rt.device
        self.latent_norm = tensors["dkv.norm"].to(dev).float().contiguous()
        if self.has_sink:
            self.sink = tensors["sink"].to(dev).float().contiguous()
        # the products into and out of the latent's space.  On the matrix cores the weights lie output-major (uv as stored,
        # [head][vdim][rank]; uk turned to [head][rank][dim]), else input-major (uk as stored, [head][dim][rank]; uv turned)
        uk = tensors["uk"].to(dev).view(self.heads, self.dim, self.rank)
        uv = tensors["uv"].to(dev).view(self.heads, self.vdim, self.rank)
        per = self.dim + self.rot
        query_stride = self.heads * per if self.q_rank else self.proj.out_features
        self.uk_on_mfma = self.rt.bf16 and ops.headwise_mfma_ok(uk, self.dim, query_stride, per)
        self.uv_on_mfma = self.rt.bf16 and ops.headwise_mfma_ok(uv, self.rank, self.heads * self.rank, self.rank)
        self.uk_t = uk.transpose(1, 2).contiguous() if self.uk_on_mfma else uk.contiguous()
        self.uv_t = uv.contiguous() if self.uv_on_mfma else uv.transpose(1, 2).contiguous()

    def weight_bytes(self) -> int:
        small = self.uk_t.numel() * self.uk_t.element_size() + self.uv_t.numel() * self.uv_t.element_size()
        return self.proj.nbytes() + (0 if self.uq is None else self.uq.nbytes()) + self.o.nbytes() + small + 4 * (
            self.rank + self.q_rank + (self.heads if self.has_sink else 0))

    def cache_spec(self) -> CacheSpec:
        return CacheSpec(1, self.key_width, self.window, key_width=self.key_width,
                         value_width=self.rank if self.on_matrix_cores else 0)

    def page_sizes(self):
        return (8, 16, 32, 64, 128) if self.on_matrix_cores else None

    def _project(self, ctx, h) -> torch.Tensor:
        y = ctx.ws.buffer("latent_proj", self.proj.out_features, torch.float32)
        self.proj.store(ctx.ws, h, y, ctx.rows)
        return y

    def _run(self, ctx, call, y, target, add: bool) -> None:
        """From the stacked product of the input (32-bit sums) to the mixer's output."""
        ws, rows = ctx.ws, ctx.rows
        table = ctx.block_tables[call.group]
        mfma = self.on_matrix_cores
        # (the matrix-core kernel takes its queries rounded to bfloat16, so they are stored that way at once)
        qa = ws.buffer("latent_q", self.heads * self.key_width, torch.bfloat16 if mfma else torch.float32)
        per = self.dim + self.rot
        cq = ws.buffer("latent_cq", self.q_rank, self.rt.act_dtype) if self.q_rank else None
        ops.latent_prep(y, self.q_off, self.dkv_off, self.latent_norm, self.eps, self.cos, self.sin, ctx.positions, ctx.row_seq,
                        table, call.k_cache, qa, rows, self.heads, self.dim, self.rot, self.rotary, self.rank, ws.page_size,
                        call.writes_cache, latent_t=call.v_cache if mfma else None, pairs=self.pairs,
                        q_latent=(self.q_norm, cq) if self.q_rank else None)
        # the unrotated query parts into the latent's space (queries out of a latent of their own: their rotated parts are
        # turned in the same launch)
        if self.q_rank:
            q = ws.buffer("latent_up_q", self.heads * per, torch.float32)
            self.uq.store(ws, cq, q, rows)
            ops.headwise_linear(q, 0, per, self.uk_t, qa, 0, self.key_width, rows, matrix_cores=self.uk_on_mfma,
                                rotate=(self.rot, self.rotary, self.pairs, self.dim, self.rank, self.cos, self.sin, ctx.positions))
        else:
            ops.headwise_linear(y, self.q_off, per, self.uk_t, qa, 0, self.key_width, rows, matrix_cores=self.uk_on_mfma)
        # (rounded where the next product would round it anyway)
        lat = ws.buffer("latent_out", self.heads * self.rank, torch.bfloat16 if mfma and self.uv_on_mfma else torch.float32)
        if mfma:
            self._attend_on_matrix_cores(ctx, call, qa, lat, table)
        else:
            many, n_many, single, n_single = _tiles(ctx, ROWS_PER_PROMPT_TILE)
            common = (call.k_cache, self.sink, lat, self.heads, self.key_width, self.rank, ws.page_size, int(self.window or 0),
                      self.scale)
            if n_many:
                ops.shared_key_attention(qa, ctx.positions, table, many, n_many, *common, 16 // ROWS_PER_PROMPT_TILE)
            if n_single:
                ops.shared_key_attention(qa, ctx.positions, table, single, n_single, *common, 16)
        vals = ws.buffer("latent_values", self.heads * self.vdim, self.rt.act_dtype)
        ops.headwise_linear(lat, 0, self.rank, self.uv_t, vals, 0, self.vdim, rows, matrix_cores=self.uv_on_mfma,
                            gate=y[:, self.gate_off:self.gate_off + self.heads] if self.has_gate else None)
        if add:
            self.o.add_into(ws, vals, target, rows)
        else:
            self.o.store(ws, vals, target, rows)

    def forward(self, ctx, call, h, residual) -> None:
        self._run(ctx, call, self._project(ctx, h), residual, True)

    def forward_out(self, ctx, call, h, out) -> None:
        self._run(ctx, call, self._project(ctx, h), out, False)

    def forward_between_norms(self, ctx, call, x, norm, norm_behind) -> bool:
        """Decode steps of few rows: the norm in front rides in the first product."""
        y = ctx.ws.buffer("latent_proj", self.proj.out_features, torch.float32)
        if not self.proj.store_normed(x, norm, y, ctx.rows):
            return False
        out = ctx.ws.buffer("sublayer_out", self.width, torch.float32)
        self._run(ctx, call, y, out, False)
        norm_behind.add_normed(ctx, out, x)
        return True

    def _attend_on_matrix_cores(self, ctx, call, qa, lat, table) -> None:
        ws = ctx.ws
        hg = self.heads_per_group
        many, n_many, single, n_single = _tiles(ctx, ops.SHARED_KEY_TILE_QUERIES // hg)
        window = int(self.window or 0)
        common = (call.k_cache, call.v_cache, self.sink, lat, self.heads, self.key_width, self.rank, ws.page_size, window, self.scale)
        if n_many:
            ops.shared_key_attention_mfma(qa, ctx.positions, table, many, n_many, *common, hg)
        if n_single:
            # Single tokens: a workgroup for every piece of keys the token can see, folded by a second launch; few tokens
            # with long contexts still fill the chip.  Prompt tiles cut their keys at the same places and fold them by the
            # same operations, so a position's bits do not depend on how it came.
            pieces = ops.shared_key_pieces(table.shape[1] * ws.page_size, window)
            # (room for the power of two from this step's single tokens up: a few sizes at most)
            tokens = 1 << max(0, n_single - 1).bit_length()
            widest = pieces if ws.max_table_width is None else ops.shared_key_pieces(ws.max_table_width * ws.page_size, window)
            partial = ws.buffer("latent_pieces", tokens * max(pieces, widest) * self.heads * (self.rank + 2), torch.float32, rows=1)
            ops.shared_key_attention_mfma(qa, ctx.positions, table, single, n_single, *common, 16, pieces, partial)
