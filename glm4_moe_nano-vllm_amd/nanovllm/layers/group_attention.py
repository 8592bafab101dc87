"""Attention with grouped heads over paged key / value caches, without rotation: chunks or a sliding window, a distance bias and a
sink per head are options (csrc/group_attn.hip).

A layer may read another layer's cache (it then has queries only): the caches are an argument of forward."""
from __future__ import annotations

import torch
from torch import nn

from nanovllm import hip_ops
from nanovllm.distributed.parallel_state import get_tp_group
from nanovllm.layers.linear import PaddedLinear


def distance_slopes(heads: int) -> torch.Tensor:
    """Slope of the distance bias per head: a geometric series from 2^(-8 / heads) to 2^-8."""
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)], dtype=torch.float32, device="cpu")


class GroupAttention(nn.Module):

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, dtype, own_kv: bool = True, window: int = 0, chunk: int = 0,
                 biased: bool = False):
        super().__init__()
        tp = get_tp_group()
        if heads % tp.world_size or kv_heads % tp.world_size:
            raise ValueError(f"{heads} heads over {kv_heads} key/value heads do not split over {tp.world_size} ranks")
        self.tp_size, self.tp_rank = tp.world_size, tp.rank
        self.heads, self.kv_heads, self.total_heads = heads // tp.world_size, kv_heads // tp.world_size, heads
        self.dim, self.vdim, self.scale, self.dtype, self.own_kv, self.window, self.chunk, self.biased = dim, vdim, scale, dtype, own_kv, window, chunk, biased
        self.dimp, self.vdimp = hip_ops.round8(dim), hip_ops.round8(vdim)
        H, G = self.heads, self.kv_heads
        self.qkv_proj = PaddedLinear(width, [self.dimp] * H + ([self.dimp] * G + [self.vdimp] * G if own_kv else []), dtype)
        self.o_proj = PaddedLinear([vdim] * H, [hip_ops.round8(width)], dtype)
        # (fp32, and what the tiled kernels do not take: one evaluation for all portions)
        self.tiled = dtype == torch.bfloat16 and scale > 0 and max(self.dimp, self.vdimp) <= hip_ops.GROUP_ATTN_MAX_DIM
        self.tokens_per_tile = max(1, hip_ops.GROUP_ATTN_ROWS // (H // G)) if self.tiled else 1
        self.tile_rows = hip_ops.group_attn_tile_rows(H, G)
        self.slope = self.sink = self.k_cache = self.v_cache = None

    def load(self, w: dict, device) -> None:
        """w: q, o; k and v unless the layer borrows a cache; sink (optional)."""
        def heads_of(t, n, size):  # this rank's heads of a head-by-head layout
            return list(t.view(n * self.tp_size, size, -1)[self.tp_rank * n: (self.tp_rank + 1) * n].to(device))

        H, G, h0 = self.heads, self.kv_heads, self.tp_rank * self.heads
        blocks = heads_of(w["q"], H, self.dim)
        if self.own_kv:
            blocks += heads_of(w["k"], G, self.dim) + heads_of(w["v"], G, self.vdim)
        self.qkv_proj.load(blocks, device)
        if "sink" in w:
            self.sink = w["sink"][h0: h0 + H].to(device=device, dtype=torch.float32).contiguous()
        if self.biased:
            self.slope = distance_slopes(self.total_heads)[h0: h0 + H].to(device).contiguous()
        self.o_proj.load([w["o"][:, h0 * self.vdim: (h0 + H) * self.vdim]], device)

    def cache_bytes_per_token(self) -> int:
        return self.kv_heads * (self.dimp + self.vdimp) * self.dtype.itemsize if self.own_kv else 0

    def allocate_cache(self, num_blocks: int, block_size: int, device) -> None:
        if self.own_kv:
            self.k_cache, self.v_cache = (torch.empty(num_blocks, self.kv_heads, block_size, d, dtype=self.dtype, device=device) for d in (self.dimp, self.vdimp))

    def forward(self, h: torch.Tensor, meta, cache: tuple | None = None) -> torch.Tensor:
        H, T, Ta = self.heads, h.shape[0], meta.Ta
        x = self.qkv_proj(h)
        nq = H * self.dimp
        kc, vc = cache or (self.k_cache, self.v_cache)
        nk = nq + self.kv_heads * self.dimp
        Ts = Ta if self.tiled else 0    # the decode kernel stores its rows' keys and values itself
        if self.own_kv and Ts < T:
            hip_ops.group_kv_store(x[Ts:], nq, nk, meta.slots[Ts:], kc, vc)
        q = x[:, :nq]
        out = torch.empty((T, H * self.vdimp), dtype=h.dtype, device=h.device)
        form = (H, self.window, self.chunk, self.scale, self.slope, self.sink)
        if not self.tiled:
            hip_ops.group_attn_plain(q, kc, vc, meta.block_tables, meta.pos, meta.seq_of, *form, out)
        else:
            if Ta:
                per = min(self.tokens_per_tile, meta.max_short)
                tok, n = meta.tiles[per]
                new = (x[:Ta, nq: nk], x[:Ta, nk:], meta.q_start, meta.slots) if self.own_kv else None
                hip_ops.group_attn_decode(q[:Ta], kc, vc, meta.block_tables, meta.pos, meta.seq_of, tok, n, per, *form, out, new=new)
            if Ta < T:
                hip_ops.group_attn_prefill(q[Ta:], kc, vc, meta.block_tables, meta.n_short, meta.long_q_start, meta.pos[Ta:],
                                           *meta.chunk_tiles[self.chunk, self.tile_rows], *form, out[Ta:])
        y = self.o_proj(out)
        if self.tp_size > 1:
            get_tp_group().all_reduce(y)
        return y
