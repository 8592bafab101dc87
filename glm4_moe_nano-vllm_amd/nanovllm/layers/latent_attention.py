"""Latent attention over a paged cache of one latent row per token, with a sliding window and a sink per head, without
positions (csrc/latent_attn.hip, csrc/window_attn.hip).

Two evaluations of the same mechanism share a step: short portions (decoded tokens above all) attend in the absorbed form over
the cached latents, long portions expand keys and values.  The step's batch says which rows are which (StepBatch.Ta)."""
from __future__ import annotations

import torch
from torch import nn

from nanovllm import hip_ops
from nanovllm.distributed.parallel_state import get_tp_group
from nanovllm.layers.linear import PaddedLinear
from nanovllm.layers.seq_norm import norm_gain


def absorb_break_even(rank: int, dim: int, vdim: int) -> int:
    """Tokens per portion up to which the absorbed form is used.  Per query token, head and visible key the absorbed form costs
    2 rank multiply-adds and the expanded one dim + vdim, plus rank (dim + vdim) for every key it expands; half the
    break-even, since the expanded kernel runs at a higher rate, within what one step can reasonably hold."""
    extra = 2 * rank - (dim + vdim)
    even = rank * (dim + vdim) / extra if extra > 0 else 1 << 30
    return int(min(128, max(16, even / 2)))


class LatentAttention(nn.Module):

    def __init__(self, width: int, heads: int, dim: int, vdim: int, rank: int, window: int, scale: float, eps: float, dtype, runs: int = 1):
        super().__init__()
        tp = get_tp_group()
        if heads % tp.world_size:
            raise ValueError(f"{heads} heads do not split over {tp.world_size} ranks")
        self.tp_size, self.tp_rank = tp.world_size, tp.rank
        self.heads = heads // tp.world_size
        self.dim, self.vdim, self.rank, self.window, self.scale, self.eps, self.dtype = dim, vdim, rank, window, scale, eps, dtype
        self.dimp, self.vdimp, self.rp = hip_ops.round8(dim), hip_ops.round8(vdim), hip_ops.round8(rank)
        H = self.heads
        self.qc_proj = PaddedLinear(width, [self.dimp] * H + [self.rp], dtype)     # query heads, raw latent
        # (fp32, and heads beyond the expanded kernel's sizes: every portion attends in the absorbed form)
        self.can_expand = dtype == torch.bfloat16 and max(self.dimp, self.vdimp) <= hip_ops.WINDOW_ATTN_MAX_DIM
        self.expand = PaddedLinear(rank, [self.dimp] * H + [self.vdimp] * H, dtype) if self.can_expand else None
        self.o_proj = PaddedLinear([vdim] * H, [hip_ops.round8(width)], dtype)
        self.tokens_per_tile = hip_ops.latent_tokens_per_tile(self.rp, H) if dtype == torch.bfloat16 else 1
        self.break_even = absorb_break_even(self.rp, self.dimp, self.vdimp)
        self.caches: list = [None] * runs
        self.runs = runs

    def load(self, w: dict, device) -> None:
        """w: q, dkv, dkv.norm, uk, uv, sink, o."""
        H, h0 = self.heads, self.tp_rank * self.heads

        def heads_of(t, size):  # this rank's heads of a head-by-head layout
            return t.view(H * self.tp_size, size, -1)[h0: h0 + H].to(device)

        q, uk, uv = heads_of(w["q"], self.dim), heads_of(w["uk"], self.dim), heads_of(w["uv"], self.vdim)
        self.qc_proj.load(list(q) + [w["dkv"]], device)
        if self.expand is not None:
            self.expand.load(list(uk) + list(uv), device)
        self.wukt = torch.zeros(H, self.rp, self.dimp, dtype=self.dtype, device=device)
        self.wukt[:, : self.rank, : self.dim] = uk.transpose(1, 2).to(self.dtype)
        self.wuv = torch.zeros(H, self.vdimp, self.rp, dtype=self.dtype, device=device)
        self.wuv[:, : self.vdim, : self.rank] = uv.to(self.dtype)
        self.c_gain = norm_gain(w["dkv.norm"], self.rp, device, zero_centred=False)
        self.sink = w["sink"][h0: h0 + H].to(device=device, dtype=torch.float32).contiguous()
        self.o_proj.load([w["o"][:, h0 * self.vdim: (h0 + H) * self.vdim]], device)

    def cache_bytes_per_token(self) -> int:
        return self.runs * self.rp * self.dtype.itemsize

    def allocate_cache(self, num_blocks: int, block_size: int, device) -> None:
        self.caches = [torch.empty(num_blocks, block_size, self.rp, dtype=self.dtype, device=device) for _ in range(self.runs)]

    def forward(self, h: torch.Tensor, meta, run: int) -> torch.Tensor:
        H, Ta, T = self.heads, meta.Ta, h.shape[0]
        cache = self.caches[run]
        qc = self.qc_proj(h)
        nq = H * self.dimp
        win = meta.windows[self.window] if Ta < T else None
        qa, c_all = hip_ops.latent_prepare(qc, nq, H, self.dimp, self.rank, self.c_gain, self.eps, meta.slots, cache, Ta, self.wukt,
                                           win.crow if win else None, win.rows if win else 0)
        out = torch.empty((T, H * self.vdimp), dtype=h.dtype, device=h.device)
        if Ta:
            tok, n = meta.tiles[min(self.tokens_per_tile, meta.max_short)]
            hip_ops.latent_attn(qa, cache, tok, n, min(self.tokens_per_tile, meta.max_short), meta.pos, meta.seq_of, meta.block_tables,
                                self.rank, self.window, self.scale, self.sink, self.wuv, out)
        if Ta < T:
            if win.hist_rows.numel():
                hip_ops.latent_gather(cache, win.hist_slots, win.hist_rows, c_all)
            kv = self.expand(c_all)
            hip_ops.window_attn_prefill(qc[Ta:, :nq], kv[:, :nq], kv[:, nq:], out[Ta:], meta.long_q_start, win.k_start, meta.long_tile_seq,
                                        meta.long_tile_off, H, self.dimp, self.vdimp, self.window, self.scale, self.sink)
        y = self.o_proj(out)
        if self.tp_size > 1:
            get_tp_group().all_reduce(y)
        return y
