"""Attention with grouped heads over paged key / value caches (csrc/group_attn.hip, csrc/group_rows.hip): chunks or a sliding window, a
distance bias and a sink per head, rotation of the first columns of a head, a soft cap on the scores, two maps per head whose results are
subtracted (differential attention), sigmoid weights over keys that are the values, and a gate on the output are options.

A layer may read another layer's cache (it then has queries only): the caches are an argument of forward.  The projections may belong to
the caller (`joint`: ParallelBlock makes them part of larger ones); `attend` is what lies between them."""
from __future__ import annotations

from dataclasses import replace

import torch
from torch import nn

from nanovllm import hip_ops
from nanovllm.distributed.parallel_state import get_tp_group
from nanovllm.layers.linear import PaddedLinear
from nanovllm.layers.rotary_embedding import HalfRotary


def distance_slopes(heads: int) -> torch.Tensor:
    """Slope of the distance bias per head: a geometric series from 2^(-8 / heads) to 2^-8."""
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)], dtype=torch.float32, device="cpu")


def map_weight(w: dict, offset: float) -> float:
    """exp(lq1 . lk1) - exp(lq2 . lk2) + offset: the factor of a layer's second map, in fp32."""
    f = {k: w[k].detach().to(device="cpu", dtype=torch.float32) for k in ("lq1", "lk1", "lq2", "lk2")}
    return float(torch.exp((f["lq1"] * f["lk1"]).sum()) - torch.exp((f["lq2"] * f["lk2"]).sum()) + offset)


class GroupAttention(nn.Module):

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, dtype, own_kv: bool = True, window: int = 0, chunk: int = 0,
                 biased: bool = False, *, joint: bool = False, runs: int = 1, eps: float = 0.0, rot: HalfRotary | None = None, cap: float = 0.0,
                 diff: float | None = None, sigmoid_kv: bool = False, temperature: tuple = (0.0, 0), gate: str | None = None):
        """rot: rotation of queries and keys; cap: soft cap; diff: two maps of `dim` columns per head, o = (1 - diff) unit_rms(o_1 - lam o_2),
        lam from learned vectors and diff; sigmoid_kv: weights sigmoid(score + bias per head), queries and keys normed over the whole
        projection, values the keys in front of their norm, queries times 1 + coef ln(floor((p + 1) / every) + 1) with temperature =
        (coef, every); gate: one per "head" or per "column" of the output, already through its sigmoid where attend reads it; runs: how often
        the layer runs in a step, each run with its own cache."""
        super().__init__()
        tp = get_tp_group()
        if heads % tp.world_size or kv_heads % tp.world_size:
            raise ValueError(f"{heads} heads over {kv_heads} key/value heads do not split over {tp.world_size} ranks")
        if sigmoid_kv and (dim != vdim or rot or diff is not None or cap or not own_kv):
            raise ValueError(f"keys of {dim} columns that are values of {vdim}, or parts that do not go together")
        self.tp_size, self.tp_rank = tp.world_size, tp.rank
        self.heads, self.kv_heads, self.total_heads, self.total_kv = heads // tp.world_size, kv_heads // tp.world_size, heads, kv_heads
        self.dim, self.vdim, self.scale, self.dtype, self.own_kv, self.window, self.chunk, self.biased = dim, vdim, scale, dtype, own_kv, window, chunk, biased
        self.eps, self.rot, self.cap, self.diff, self.sigmoid_kv, self.temperature, self.gate, self.runs = eps, rot, cap, diff, sigmoid_kv, temperature, gate, runs
        self.maps = 1 if diff is None else 2
        self.dimp, self.vdimp = hip_ops.round8(dim), hip_ops.round8(vdim)
        self.dk = self.maps * self.dimp            # columns of a key row
        H, G = self.heads, self.kv_heads
        # (norms over the whole projection need all heads on every rank)
        self.q_heads, self.k_heads = (heads, kv_heads) if sigmoid_kv else (H, G)
        self.k_off = self.q_heads * self.dk
        self.v_off = self.k_off + (self.k_heads * self.dk if own_kv else 0)
        self.g_off = self.v_off + (G * self.vdimp if own_kv and not sigmoid_kv else 0)
        self.in_sizes = [self.dimp] * (self.q_heads * self.maps) + ([self.dimp] * (self.k_heads * self.maps) if own_kv else [])
        self.in_sizes += [self.vdimp] * G if own_kv and not sigmoid_kv else []
        self.in_sizes += {None: [], "head": [hip_ops.round8(H)], "column": [self.vdimp] * H}[gate]
        self.out_sizes = [vdim] * H
        self.joint = joint
        if not joint:
            assert gate is None, "a gate needs its activation in the caller's projection"
            self.qkv_proj = PaddedLinear(width, self.in_sizes, dtype)
            self.o_proj = PaddedLinear(self.out_sizes, [hip_ops.round8(width)], dtype)
        # (fp32, and what the tiled kernels do not take: one evaluation for all portions)
        self.tiled = dtype == torch.bfloat16 and scale > 0 and max(self.dk, self.vdimp) <= hip_ops.GROUP_ATTN_MAX_DIM and (not cap or self.maps == 2)
        self.tokens_per_tile = max(1, hip_ops.group_attn_rows(self.maps) // (H // G)) if self.tiled else 1
        self.tile_rows = hip_ops.group_attn_tile_rows(H, G, self.maps)
        self.slope = self.sink = self.gain = None
        self.parts = hip_ops.NO_PARTS
        self.caches: list = [(None, None, None)] * runs    # keys, values, factors of the keys

    @property
    def k_cache(self):
        return self.caches[0][0]

    @property
    def v_cache(self):
        return self.caches[0][1]

    # ------------------------------------------------------------------ weights
    def in_blocks(self, w: dict, device) -> list[torch.Tensor]:
        """This rank's rows of the input projection, a block per entry of in_sizes.  w: q; k and v unless the layer borrows a cache or its
        values are its keys; g if there is a gate."""
        def heads_of(t, n, size):  # this rank's heads of a head-by-head layout
            return list(t.view(n * self.tp_size, size, -1)[self.tp_rank * n: (self.tp_rank + 1) * n].to(device))

        H, G, m = self.heads, self.kv_heads, self.maps
        if self.sigmoid_kv:
            blocks = list(w["q"].view(self.q_heads, self.dim, -1).to(device)) + list(w["k"].view(self.k_heads, self.dim, -1).to(device))
        else:
            blocks = heads_of(w["q"], H * m, self.dim)
            if self.own_kv:
                blocks += heads_of(w["k"], G * m, self.dim) + heads_of(w["v"], G, self.vdim)
        if self.gate == "head":
            blocks += [torch.cat(heads_of(w["g"], H, 1))]
        elif self.gate == "column":
            blocks += heads_of(w["g"], H, self.vdim)
        return blocks

    def out_block(self, w: dict) -> torch.Tensor:
        """This rank's columns of the output projection."""
        h0 = self.tp_rank * self.heads
        return w["o"][:, h0 * self.vdim: (h0 + self.heads) * self.vdim]

    def load_small(self, w: dict, device) -> None:
        """What is no projection.  w: sink (optional); lq1, lk1, lq2, lk2 with two maps; q.norm, k.norm, pb with sigmoid weights."""
        H, h0 = self.heads, self.tp_rank * self.heads
        f32 = lambda t: t.to(device=device, dtype=torch.float32)  # noqa: E731
        if "sink" in w:
            self.sink = f32(w["sink"][h0: h0 + H]).contiguous()
        if self.biased:
            self.slope = distance_slopes(self.total_heads)[h0: h0 + H].to(device).contiguous()
        self.parts = hip_ops.GroupParts(cap=self.cap, maps=self.maps, eps=self.eps, gate_cols=self.gate == "column")
        if self.maps == 2:
            self.parts = replace(self.parts, lam=map_weight(w, self.diff), post=1.0 - self.diff, vn=self.vdim)
        if self.sigmoid_kv:
            self.parts = replace(self.parts, sigmoid=True, bias=f32(w["pb"][h0: h0 + H]).contiguous())
            # the keys' gains meet the queries' in the products of a score: a query carries both
            R = self.q_heads // self.k_heads
            both = f32(w["q.norm"]).view(self.k_heads, R, self.dim) * f32(w["k.norm"]).view(self.k_heads, 1, self.dim)
            self.gain = torch.zeros(self.q_heads, self.dimp, dtype=torch.float32, device=device)
            self.gain[:, : self.dim] = both.reshape(self.q_heads, self.dim)
            self.gain = self.gain.view(-1)
        if self.rot is not None:
            self.rot.prepare(torch.empty(0, device=device).device)

    def load(self, w: dict, device) -> None:
        """w: q, o; k and v unless the layer borrows a cache; and load_small's."""
        self.load_small(w, device)
        self.qkv_proj.load(self.in_blocks(w, device), device)
        self.o_proj.load([self.out_block(w)], device)

    # ------------------------------------------------------------------ cache
    def cache_bytes_per_token(self) -> int:
        if not self.own_kv:
            return 0
        row = self.kv_heads * self.dk * self.dtype.itemsize + 4 if self.sigmoid_kv else self.kv_heads * (self.dk + self.vdimp) * self.dtype.itemsize
        return self.runs * row

    def allocate_cache(self, num_blocks: int, block_size: int, device) -> None:
        def rows(d):
            return torch.empty(num_blocks, self.kv_heads, block_size, d, dtype=self.dtype, device=device)

        for i in range(self.runs if self.own_kv else 0):
            k = rows(self.dk)
            if self.sigmoid_kv:
                self.caches[i] = (k, k, torch.empty(num_blocks, block_size, dtype=torch.float32, device=device))
            else:
                self.caches[i] = (k, rows(self.vdimp), None)

    # ------------------------------------------------------------------ step
    def attend(self, x: torch.Tensor, out: torch.Tensor, meta, cache: tuple | None = None, run: int = 0, cs: torch.Tensor | None = None) -> None:
        """From the projection's rows x (columns as in_sizes) to the heads' outputs.  cache: another layer's (keys, values); cs: the step's
        rotation table of self.rot."""
        H, T, Ta = self.heads, x.shape[0], meta.Ta
        kc, vc, ks = (*cache, None) if cache else self.caches[run]
        nq, nk, nv = self.k_off, self.v_off, self.v_off + self.kv_heads * self.vdimp
        stores = False                      # the decode kernel stores its rows' keys and values itself
        if self.sigmoid_kv:
            hip_ops.group_norm_store(x, 0, self.k_off, self.gain, self.q_heads * self.dim, self.k_heads * self.dk, self.k_heads * self.dim, self.tp_rank * self.kv_heads, self.eps,
                                     meta.pos, meta.slots, kc, ks, self.temperature)
            q = x[:, self.tp_rank * H * self.dk: (self.tp_rank + 1) * H * self.dk]
        else:
            q, stores = x[:, :nq], self.own_kv and self.tiled and self.maps == 1 and self.rot is None
            if self.rot is not None:
                hip_ops.group_rotate_store(x, 0, self.k_off, self.v_off, H, self.maps, self.rot.dims, cs, meta.slots, kc, vc)
            elif self.own_kv and (Ts := Ta if stores else 0) < T:
                hip_ops.group_kv_store(x[Ts:], nq, nk, meta.slots[Ts:], kc, vc)
        gate = x[:, self.g_off:] if self.gate else None
        parts = self.parts if ks is None and gate is None else replace(self.parts, kscale=ks, gate=gate)
        form = (H, self.window, self.chunk, self.scale, self.slope, self.sink)
        if not self.tiled:
            hip_ops.group_attn_plain(q, kc, vc, meta.block_tables, meta.pos, meta.seq_of, *form, out, parts=parts)
            return
        if Ta:
            per = min(self.tokens_per_tile, meta.max_short)
            tok, n = meta.tiles[per]
            new = (x[:Ta, nq: nk], x[:Ta, nk: nv], meta.q_start, meta.slots) if stores else None
            hip_ops.group_attn_decode(q[:Ta], kc, vc, meta.block_tables, meta.pos, meta.seq_of, tok, n, per, *form, out, new=new, parts=parts)
        if Ta < T:
            if gate is not None:
                parts = replace(parts, gate=gate[Ta:])
            hip_ops.group_attn_prefill(q[Ta:], kc, vc, meta.block_tables, meta.n_short, meta.long_q_start, meta.pos[Ta:],
                                       *meta.chunk_tiles[self.chunk, self.tile_rows], *form, out[Ta:], parts=parts)

    def forward(self, h: torch.Tensor, meta, cache: tuple | None = None, run: int = 0, cs: torch.Tensor | None = None) -> torch.Tensor:
        x = self.qkv_proj(h)
        out = torch.empty((h.shape[0], self.heads * self.vdimp), dtype=h.dtype, device=h.device)
        self.attend(x, out, meta, cache, run, cs)
        y = self.o_proj(out)
        if self.tp_size > 1:
            get_tp_group().all_reduce(y)
        return y
