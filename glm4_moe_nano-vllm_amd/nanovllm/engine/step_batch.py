"""One step's inputs for models that run portions of prompts beside single decoded tokens: what every row is (token, position,
cache row), which rows belong to which sequence, where the recurrent state of a sequence is read and written, and the work
lists of the attention kernels.  Everything the kernels read is packed into ONE int32 buffer: one copy to the device per step,
and a captured step replays over a fixed buffer of the same layout.

Rows are ordered short portions first (they take the kernels for few rows per sequence), then long ones; results go back in chunk order."""
from __future__ import annotations

from dataclasses import dataclass, field
from types import SimpleNamespace

import numpy as np
import torch


@dataclass
class Chunk:
    """A portion of one sequence: the next `tokens` from position `start`, with the cache blocks and the state slot it holds."""
    tokens: list
    start: int
    block_table: list
    state_in: int
    state_out: int
    want: list = field(default_factory=list)   # places among `tokens` whose logits are asked for
    temperature: float = 0.0


class _Packer:
    """int32 arrays behind one another (16-byte aligned), viewed again from one device tensor."""

    def __init__(self):
        self.parts, self.offsets, self.n = [], [], 0

    def add(self, a) -> int:
        a = np.ascontiguousarray(a, dtype=np.int32)
        self.parts.append(a)
        self.offsets.append(self.n)
        self.n += (a.size + 3) // 4 * 4
        return len(self.parts) - 1

    def host(self) -> np.ndarray:
        buf = np.zeros(max(self.n, 4), dtype=np.int32)
        for o, a in zip(self.offsets, self.parts):
            buf[o: o + a.size] = a.reshape(-1)
        return buf

    def view(self, buf: torch.Tensor, i: int) -> torch.Tensor:
        a = self.parts[i]
        return buf[self.offsets[i]: self.offsets[i] + a.size].view(a.shape)


LONG_TILE = 128  # query rows of a long portion per workgroup (csrc/window_attn.hip, csrc/group_attn.hip)


class StepBatch(SimpleNamespace):
    """Device views: ids int64 [T]; pos, seq_of, slots [T]; q_start [S+1]; state_in, state_out [S]; block_tables [S, width];
    want [n]; tiles {tokens per tile: (first row, rows)}; Ta rows of n_short short portions in front, max_short; and, if Ta < T: long_q_start, long_tile_seq,
    long_tile_off, chunk_tiles {(chunk, rows): tiles of that many rows}, windows {size: (rows, k_start, crow, hist_slots, hist_rows)}."""


def build_step(chunks: list[Chunk], spec, block_size: int, pad_rows: int = 0, table_width: int = 0):
    """spec: the model (windows, tile_sizes, max_short_portion; chunk_tiles if it wants some).  pad_rows > 0: a decode step of exactly that many rows, the
    missing ones unused (position -1), with block tables of table_width columns.
    Returns (host int32 buffer, function device buffer -> StepBatch, order of the wanted rows in chunk order)."""
    limit = spec.max_short_portion
    order = sorted(range(len(chunks)), key=lambda i: (len(chunks[i].tokens) > limit, i))
    seqs = [chunks[i] for i in order]
    lens = np.array([len(c.tokens) for c in seqs], dtype=np.int64)
    if pad_rows:
        assert (lens == 1).all() and len(seqs) <= pad_rows
    n_pad = pad_rows - len(seqs) if pad_rows else 0
    S = len(seqs) + n_pad
    starts = np.array([c.start for c in seqs], dtype=np.int64)
    all_lens = np.concatenate([lens, np.ones(n_pad, np.int64)])
    q_start = np.concatenate([[0], np.cumsum(all_lens)])
    T = int(q_start[-1])
    seq_of = np.repeat(np.arange(S), all_lens)
    within = np.arange(T) - q_start[seq_of]
    pos = np.concatenate([starts, np.full(n_pad, -1)])[seq_of] + within
    width = max([table_width] + [len(c.block_table) for c in seqs])
    bt = np.full((S, width), -1, dtype=np.int64)
    for s, c in enumerate(seqs):
        bt[s, : len(c.block_table)] = c.block_table
    used = pos >= 0
    slots = np.where(used, bt[seq_of, np.maximum(pos, 0) // block_size] * block_size + pos % block_size, -1)
    assert not used.any() or slots[used].min() >= 0, "a token without a cache block"
    ids = np.concatenate([np.concatenate([np.asarray(c.tokens, dtype=np.int64) for c in seqs]) if seqs else np.zeros(0, np.int64),
                          np.zeros(n_pad, np.int64)])

    n_short = int((all_lens <= limit).sum())
    Ta = int(q_start[n_short])
    max_short = int(all_lens[:n_short].max()) if n_short else 1
    pk = _Packer()
    f = {"ids": pk.add(ids.view(np.int32).reshape(-1)), "pos": pk.add(pos), "seq_of": pk.add(seq_of), "slots": pk.add(slots),
         "q_start": pk.add(q_start),
         "state_in": pk.add([c.state_in for c in seqs] + [0] * n_pad), "state_out": pk.add([c.state_out for c in seqs] + [-1] * n_pad),
         "block_tables": pk.add(bt)}
    first_row = {i: int(q_start[s]) for s, i in enumerate(order)}
    want = [first_row[i] + w for i, c in enumerate(chunks) for w in c.want]
    f["want"] = pk.add(np.arange(T) if pad_rows else want)

    tiles = {}
    for size in sorted({min(t, max_short) for t in spec.tile_sizes}):
        if max_short == 1:
            tok, cnt = np.arange(Ta), np.ones(Ta, np.int64)
        else:
            n_tiles = -(-all_lens[:n_short] // size)
            tseq = np.repeat(np.arange(n_short), n_tiles)
            k = np.arange(len(tseq)) - np.repeat(np.cumsum(n_tiles) - n_tiles, n_tiles)
            tok = q_start[tseq] + k * size
            cnt = np.minimum(size, all_lens[tseq] - k * size)
        tiles[size] = (pk.add(tok), pk.add(cnt))

    longs, windows, chunk_tiles = None, {}, {}
    if Ta < T:
        L = np.arange(n_short, S)
        n_tiles = -(-all_lens[L] // LONG_TILE)
        tseq = np.repeat(np.arange(len(L)), n_tiles)
        k = np.arange(len(tseq)) - np.repeat(np.cumsum(n_tiles) - n_tiles, n_tiles)
        tseq, k = tseq[::-1], k[::-1]   # a portion's last rows see the most keys: they start first, over all portions
        keys = np.minimum(starts[n_short:][tseq] + (k + 1) * LONG_TILE, max(spec.windows, default=1 << 30))
        o = np.argsort(-keys, kind="stable")
        tseq, k = tseq[o], k[o]
        longs = (pk.add(q_start[n_short:] - Ta), pk.add(tseq), pk.add(k * LONG_TILE))
        for c, rows in getattr(spec, "chunk_tiles", ()):            # tiles for attention over chunks, the ones with the most keys first
            m = -(-all_lens[L] // rows)
            tseq = np.repeat(np.arange(len(L)), m)
            off = (np.arange(len(tseq)) - np.repeat(np.cumsum(m) - m, m)) * rows
            last = starts[n_short:][tseq] + np.minimum(off + rows, all_lens[L][tseq]) - 1   # position of a tile's last row
            o = np.argsort(-(last % c if c else last), kind="stable")
            chunk_tiles[c, rows] = (pk.add(tseq[o]), pk.add(off[o]))
        for w in spec.windows:
            hist = np.minimum(starts[n_short:], w - 1)           # tokens in front of the portion that its first row still sees
            k_start = np.concatenate([[0], np.cumsum(hist + all_lens[L])])
            crow = np.full(T, -1)
            ls = seq_of[Ta:] - n_short
            crow[Ta:] = k_start[ls] + hist[ls] + within[Ta:]
            hseq = np.repeat(np.arange(len(L)), hist)
            hk = np.arange(len(hseq)) - np.repeat(np.cumsum(hist) - hist, hist)
            hpos = starts[n_short:][hseq] - hist[hseq] + hk
            hslots = bt[n_short + hseq, hpos // block_size] * block_size + hpos % block_size
            windows[w] = (int(k_start[-1]), pk.add(k_start), pk.add(crow), pk.add(hslots), pk.add(k_start[hseq] + hk))

    def on_device(buf: torch.Tensor) -> StepBatch:
        v = lambda i: pk.view(buf, i)  # noqa: E731
        b = StepBatch(**{name: v(i) for name, i in f.items()}, Ta=Ta, n_short=n_short, max_short=max_short,
                      tiles={s: (v(a), v(c)) for s, (a, c) in tiles.items()}, windows={})
        b.ids = b.ids.view(torch.int64)
        if longs is not None:
            b.long_q_start, b.long_tile_seq, b.long_tile_off = (v(i) for i in longs)
            b.chunk_tiles = {k: (v(q), v(o)) for k, (q, o) in chunk_tiles.items()}
            b.windows = {w: SimpleNamespace(rows=n, k_start=v(a), crow=v(c), hist_slots=v(h), hist_rows=v(r))
                         for w, (n, a, c, h, r) in windows.items()}
        return b

    return pk.host(), on_device, [first_row[i] for i in range(len(chunks))]
