"""Napadra: a decoder whose residual is several parallel 32-bit streams with learned mixing around every sublayer, a token shift in
front of every mixer, mixers that are either chunked attention with grouped heads, a distance bias and sinks (some layers reading
another layer's cache) or a gated matrix memory, clamped gated feed-forwards in some layers, and sinusoidal positions.

The model runs StepBatch inputs (engine/step_batch.py): any mixture of prompt portions and decoded tokens."""
from __future__ import annotations

import torch
import torch.nn as nn

from nanovllm import hip_ops
from nanovllm.layers.dense_mlp import GatedMLP
from nanovllm.layers.group_attention import GroupAttention
from nanovllm.layers.matrix_memory import MatrixMemory
from nanovllm.layers.stream_norm import StreamHead, StreamSublayer
from nanovllm.utils.loader import load_prefixed

MAX_SHORT = 16          # longest portion that takes the kernels for few rows per sequence
SINUSOID_BASE = 10000.0


class NapadraLayer(nn.Module):

    def __init__(self, cfg, spec):
        super().__init__()
        self.spec, dt, w = spec, cfg.torch_dtype, cfg.hidden_size

        def sub(shifted):
            return StreamSublayer(w, cfg.streams, cfg.rms_norm_eps, cfg.residual_mult, shifted)

        self.sub1, self.sub2, self.mlp = sub(True), None, None
        if spec.type == "attention":
            self.mixer = GroupAttention(w, spec.heads, spec.kv_heads, spec.dim, spec.vdim, spec.scale, dt, own_kv=spec.kv_from is None, chunk=spec.chunk, biased=True)
        else:
            self.mixer = MatrixMemory(w, spec.heads, spec.dim, spec.vdim, spec.gate_cap, cfg.rms_norm_eps, dt)
        if spec.mlp is not None:
            self.sub2, self.mlp = sub(False), GatedMLP(w, spec.ff, spec.limit, dt)

    def load_from(self, fetch, prefix: str, device) -> None:
        t = {k[len(prefix) + 1:]: v for k, v in fetch(prefix).items()}
        if not t:
            raise ValueError(f"no tensors under '{prefix}'")
        part = lambda p: {k[len(p):]: v for k, v in t.items() if k.startswith(p)}  # noqa: E731
        for q, s in ((1, self.sub1), (2, self.sub2)):
            if s is not None:
                s.load(t[f"norm{q}"], t[f"ls{q}"], t[f"hc{q}.in"], t[f"hc{q}.out"], t[f"hc{q}.mix"], t["shift"] if q == 1 else None, device)
        self.mixer.load(part("mix."), device)
        if self.mlp is not None:
            self.mlp.load(part("mlp."), device)

    def stateful(self):
        return [self.sub1, self.mixer] if isinstance(self.mixer, MatrixMemory) else [self.sub1]


class NapadraForCausalLM(nn.Module):

    def __init__(self, config):
        super().__init__()
        self.config = config
        self.dtype = config.torch_dtype
        self.layers = nn.ModuleList([NapadraLayer(config, s) for s in config.layers])
        self.final = StreamHead(config.hidden_size, config.streams, config.rms_norm_eps)
        self.embed = self.head = self.freq = None

    # ------------------------------------------------------------------ weights
    def load_weights(self, path: str) -> None:
        self.load_from(lambda prefix: load_prefixed(path, prefix))

    def load_from(self, fetch) -> None:
        """fetch(prefix) -> the tensors `prefix` and `prefix.*` of a checkpoint, by full name."""
        cfg, dev = self.config, torch.empty(0).device  # the engine builds models under torch.device(...)
        V, w, wp = cfg.vocab_size, cfg.hidden_size, cfg.padded_width

        def need(name):
            t = fetch(name).get(name)
            if t is None:
                raise ValueError(f"'{name}' not found in the checkpoint")
            return t

        def table(name):
            t = hip_ops.padded_weight(hip_ops.round8(V), wp, dtype=self.dtype, device=dev)
            t.zero_()
            t[:V, :w] = need(name).to(device=dev, dtype=self.dtype)
            return t

        self.embed, self.head = table("embed"), table("head")
        i = torch.arange(wp // 2, dtype=torch.float64, device="cpu")
        self.freq = (SINUSOID_BASE ** (-2.0 * i / w)).to(dev)
        self.final.load(need("final.norm"), dev)
        for i, layer in enumerate(self.layers):
            layer.load_from(fetch, f"l{i}", dev)

    # ------------------------------------------------------------------ cache and state
    windows = ()            # no kernel of this model wants a step's history gathered

    @property
    def _attention(self):
        return [layer.mixer for layer in self.layers if isinstance(layer.mixer, GroupAttention)]

    @property
    def chunk_tiles(self) -> list[tuple]:
        return sorted({(m.chunk, m.tile_rows) for m in self._attention})

    @property
    def tile_sizes(self) -> list[int]:
        return sorted({m.tokens_per_tile for m in self._attention})

    @property
    def max_short_portion(self) -> int:
        """Longest portion of a sequence that takes the kernels for few rows (all of them in fp32)."""
        return MAX_SHORT if self.dtype == torch.bfloat16 else 1 << 30

    def cache_bytes_per_token(self) -> int:
        return sum(m.cache_bytes_per_token() for m in self._attention)

    def state_bytes_per_slot(self) -> int:
        return 2 * sum(s.state_bytes() for layer in self.layers for s in layer.stateful())

    def allocate(self, num_blocks: int, block_size: int, num_slots: int, device) -> None:
        for m in self._attention:
            m.allocate_cache(num_blocks, block_size, device)
        for layer in self.layers:
            for s in layer.stateful():
                s.allocate_state(2 * num_slots, device)

    # ------------------------------------------------------------------ step
    def _mix(self, layer, h, meta):
        j = getattr(layer.spec, "kv_from", None)
        if j is None:
            return layer.mixer(h, meta)
        src = self.layers[j].mixer
        return layer.mixer(h, meta, cache=(src.k_cache, src.v_cache))

    def forward(self, meta, residual_tap: list | None = None) -> torch.Tensor:
        """fp32 logits [meta.want_rows, vocab] of the wanted rows of a step.  residual_tap (a list) receives the sum of the
        streams [T, width] after every layer."""
        cfg, dt = self.config, self.dtype
        x = hip_ops.embed_rows(meta.ids, self.embed[:, : cfg.hidden_size], cfg.padded_width, pos=meta.pos, freq=self.freq)   # stands for all streams
        finished = y = None          # the sublayer whose output y is not yet in x
        for layer in self.layers:
            x, h = layer.sub1.enter(x, finished, y, meta, dt)
            y, finished = self._mix(layer, h, meta), layer.sub1
            if layer.mlp is not None:
                x, h = layer.sub2.enter(x, finished, y, meta, dt)
                y, finished = layer.mlp(h), layer.sub2
            if residual_tap is not None:
                residual_tap.append(finished.leave(x, y).sum(1)[:, : cfg.hidden_size])
        if meta.want.numel() == 0:
            return torch.empty((0, cfg.vocab_size), dtype=torch.float32, device=x.device)
        h = self.final(x, finished, y, meta.want, dt)
        return hip_ops.linear_act(h, self.head, out_f32=True)[:, : cfg.vocab_size]
