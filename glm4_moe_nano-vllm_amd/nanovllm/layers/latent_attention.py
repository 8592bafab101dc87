"""Latent attention over a paged cache of one latent row per token, with a sink per head, with or without a sliding window, a rotated
key part that all heads share (cached behind the latent), queries that go through a latent of their own, and an output gate
(csrc/latent_attn.hip, csrc/window_attn.hip).

Two evaluations of the same mechanism share a step: short portions (decoded tokens above all) attend in the absorbed form over
the cached latents, long portions expand keys and values.  The step's batch says which rows are which (StepBatch.Ta)."""
from __future__ import annotations

import torch
from torch import nn

from nanovllm import hip_ops
from nanovllm.distributed.parallel_state import get_tp_group
from nanovllm.layers.linear import PaddedLinear
from nanovllm.layers.rotary_embedding import PairRotary
from nanovllm.layers.seq_norm import norm_gain


def absorb_break_even(rank: int, dim: int, vdim: int) -> int:
    """Tokens per portion up to which the absorbed form is used.  Per query token, head and visible key the absorbed form costs
    2 rank multiply-adds and the expanded one dim + vdim, plus rank (dim + vdim) for every key it expands; half the
    break-even, since the expanded kernel runs at a higher rate, within what one step can reasonably hold."""
    extra = 2 * rank - (dim + vdim)
    even = rank * (dim + vdim) / extra if extra > 0 else 1 << 30
    return int(min(128, max(16, even / 2)))


class LatentAttention(nn.Module):

    def __init__(self, width: int, heads: int, dim: int, vdim: int, rank: int, window: int, scale: float, eps: float, dtype, runs: int = 1,
                 q_rank: int | None = None, rot_dim: int = 0, rot: PairRotary | None = None, gated: bool = False):
        """q_rank: size of the queries' latent (None: queries straight from the input); rot_dim: rotated columns of a head behind the
        `dim` unrotated ones, turned by `rot`; gated: sigmoid gate on the heads, projected from the input."""
        super().__init__()
        tp = get_tp_group()
        if heads % tp.world_size:
            raise ValueError(f"{heads} heads do not split over {tp.world_size} ranks")
        self.tp_size, self.tp_rank = tp.world_size, tp.rank
        self.heads = heads // tp.world_size
        self.dim, self.vdim, self.rank, self.window, self.scale, self.eps, self.dtype = dim, vdim, rank, window, scale, eps, dtype
        self.dimp, self.vdimp, self.rp = hip_ops.round8(dim), hip_ops.round8(vdim), hip_ops.round8(rank)
        self.q_rank, self.rot_dim, self.rotp, self.rot, self.gated = q_rank, rot_dim, hip_ops.round8(rot_dim), rot, gated
        H = self.heads
        self.rc = self.rp + self.rotp                   # columns of a cache row
        head = [self.dimp] + ([self.rotp] if rot_dim else [])
        # queries (heads, or their raw latent), raw latent, raw rotated key part, gate
        queries = head * H if q_rank is None else [hip_ops.round8(q_rank)]
        self.c_off = sum(queries)
        self.qc_proj = PaddedLinear(width, queries + [self.rp] + ([self.rotp] if rot_dim else []) + ([self.vdimp] * H if gated else []), dtype)
        self.g_off = self.c_off + self.rc
        self.act = (hip_ops.ACT_GATE, float(self.g_off), 0.0) if gated else hip_ops.NO_ACT
        self.uq_proj = PaddedLinear(q_rank, head * H, dtype) if q_rank is not None else None
        # (fp32, and heads beyond the expanded kernel's sizes: every portion attends in the absorbed form)
        self.can_expand = dtype == torch.bfloat16 and max(self.dimp + self.rotp, self.vdimp) <= hip_ops.WINDOW_ATTN_MAX_DIM
        self.expand = PaddedLinear(rank, [self.dimp] * H + [self.vdimp] * H, dtype) if self.can_expand else None
        self.o_proj = PaddedLinear([vdim] * H, [hip_ops.round8(width)], dtype)
        self.tokens_per_tile = hip_ops.latent_tokens_per_tile(self.rc, H) if dtype == torch.bfloat16 else 1
        self.break_even = absorb_break_even(self.rp, self.dimp, self.vdimp)
        self.caches: list = [None] * runs
        self.runs = runs

    def load(self, w: dict, device) -> None:
        """w: q or dq, dq.norm, uq; dkv, dkv.norm, uk, uv, sink, o; g if there is a gate."""
        H, h0 = self.heads, self.tp_rank * self.heads

        def heads_of(t, size):  # this rank's heads of a head-by-head layout
            return t.view(H * self.tp_size, size, -1)[h0: h0 + H].to(device)

        uk, uv = heads_of(w["uk"], self.dim), heads_of(w["uv"], self.vdim)
        q = heads_of(w["q" if self.q_rank is None else "uq"], self.dim + self.rot_dim)
        blocks = [b for t in q for b in ((t[: self.dim], t[self.dim:]) if self.rot_dim else (t,))]
        if self.q_rank is not None:
            self.uq_proj.load(blocks, device)
            self.cq_gain = norm_gain(w["dq.norm"], hip_ops.round8(self.q_rank), device, zero_centred=False)
            blocks = [w["dq"]]
        assert w["dkv"].shape[0] == self.rank + self.rot_dim
        blocks += [w["dkv"][: self.rank]] + ([w["dkv"][self.rank:]] if self.rot_dim else [])
        self.qc_proj.load(blocks + (list(heads_of(w["g"], self.vdim)) if self.gated else []), device)
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
        return self.runs * self.rc * self.dtype.itemsize

    def allocate_cache(self, num_blocks: int, block_size: int, device) -> None:
        self.caches = [torch.empty(num_blocks, block_size, self.rc, dtype=self.dtype, device=device) for _ in range(self.runs)]

    def _queries(self, h: torch.Tensor, meta, cache, win, cs):
        """Projections, norms, cache store.  Returns (query rows, absorbed queries of the first Ta rows, latent rows for the expanded
        form, gate rows)."""
        H, Ta, T = self.heads, meta.Ta, h.shape[0]
        x = self.qc_proj(h, act=self.act)
        gate = x[:, self.g_off:] if self.gated else None
        crow, n_crows = (win.crow, win.rows) if win else (None, 0)
        if self.q_rank is None and not self.rotp:
            qa, c_all = hip_ops.latent_prepare(x, self.c_off, H, self.dimp, self.rank, self.c_gain, self.eps, meta.slots, cache, Ta, self.wukt, crow, n_crows)
            return x[:, : self.c_off], qa, c_all, gate
        query = (0, self.q_rank, self.cq_gain) if self.q_rank is not None else None
        cq, c_all = hip_ops.latent_rows(x, self.c_off, self.rank, self.c_gain, cs, self.eps, meta.slots, cache, query, crow, n_crows)
        q = self.uq_proj(cq) if query else x[:, : self.c_off]
        return q, hip_ops.latent_absorb(q[:Ta], H, self.dimp, cs, self.wukt, self.rotp) if Ta else None, c_all, gate

    def forward(self, h: torch.Tensor, meta, run: int = 0, cs: torch.Tensor | None = None) -> torch.Tensor:
        """cs: the step's rotation table of self.rot (PairRotary.table)."""
        H, Ta, T = self.heads, meta.Ta, h.shape[0]
        cache = self.caches[run]
        win = meta.windows[self.window] if Ta < T else None
        q, qa, c_all, gate = self._queries(h, meta, cache, win, cs)
        out = torch.empty((T, H * self.vdimp), dtype=h.dtype, device=h.device)
        if Ta:
            tok, n = meta.tiles[min(self.tokens_per_tile, meta.max_short)]
            hip_ops.latent_attn(qa, cache, tok, n, min(self.tokens_per_tile, meta.max_short), meta.pos, meta.seq_of, meta.block_tables,
                                self.window, self.scale, self.sink, self.wuv, out, gate=gate)
        if Ta < T:
            if win.hist_rows.numel():
                hip_ops.latent_gather(cache, win.hist_slots, win.hist_rows, c_all)
            kv, nk = self.expand(c_all[:, : self.rp]), H * self.dimp
            rotated = dict(kr=c_all[:, self.rp:], cs=cs[Ta:]) if self.rotp else {}
            hip_ops.window_attn_prefill(q[Ta:], kv[:, :nk], kv[:, nk:], out[Ta:], meta.long_q_start, win.k_start, meta.long_tile_seq, meta.long_tile_off, H,
                                        self.dimp + self.rotp, self.vdimp, self.window, self.scale, self.sink, gate=gate[Ta:] if gate is not None else None, **rotated)
        y = self.o_proj(out)
        if self.tp_size > 1:
            get_tp_group().all_reduce(y)
        return y
