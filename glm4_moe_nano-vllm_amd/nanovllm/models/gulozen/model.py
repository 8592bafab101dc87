"""Gulozen: a decoder whose sublayers read the 32-bit residual as it is and are closed by norms in groups, with a short convolution in
front of every mixer, mixers that are latent attention (queries through a latent, a rotated key part with YaRN's scaling, sinks, an output
gate) or linear attention with a constant decay per head, feed-forwards of softmax-routed experts in some layers, and a learned average over
the results of all layers so far behind every layer.

The model runs StepBatch inputs (engine/step_batch.py): any mixture of prompt portions and decoded tokens."""
from __future__ import annotations

import torch
import torch.nn as nn

from nanovllm import hip_ops
from nanovllm.engine.key_reach import EVERYTHING
from nanovllm.layers.depth_norm import CausalTaps, DepthResidual
from nanovllm.layers.expert_mlp import ExpertMLP
from nanovllm.layers.latent_attention import LatentAttention
from nanovllm.layers.linear_attention import LinearAttention
from nanovllm.layers.rotary_embedding import PairRotary
from nanovllm.layers.seq_norm import norm_gain
from nanovllm.utils.loader import load_prefixed

MAX_SHORT = 16          # longest portion that takes the kernels for few rows per sequence, in a model without attention


class GulozenLayer(nn.Module):

    def __init__(self, cfg, spec):
        super().__init__()
        self.spec, dt, w = spec, cfg.torch_dtype, cfg.hidden_size
        self.taps, self.mlp, self.g_post1, self.g_post2 = CausalTaps(w, cfg.conv_taps), None, None, None
        if spec.type == "latent_attention":
            rot = PairRotary(spec.rot_dim, spec.rot_pairs_dim, spec.rot_base, spec.rot_scaling)
            self.mixer = LatentAttention(w, spec.heads, spec.dim, spec.vdim, spec.kv_rank, EVERYTHING, spec.scale, cfg.rms_norm_eps, dt,
                                         q_rank=spec.q_rank, rot_dim=spec.rot_dim, rot=rot, gated=True)
        else:
            self.mixer = LinearAttention(w, spec.heads, spec.dim, spec.vdim, spec.decay, cfg.rms_norm_eps, dt)
        if spec.mlp is not None:
            self.mlp = ExpertMLP(w, spec.ff, spec.experts, spec.top, dt)

    def load_from(self, fetch, prefix: str, device) -> torch.Tensor:
        """Loads the layer; returns the coefficients of the average behind it."""
        t = {k[len(prefix) + 1:]: v for k, v in fetch(prefix).items()}
        if not t:
            raise ValueError(f"no tensors under '{prefix}'")
        part = lambda p: {k[len(p):]: v for k, v in t.items() if k.startswith(p)}  # noqa: E731
        self.taps.load(t["canon1"], device)
        self.mixer.load(part("mix."), device)
        self.g_post1 = norm_gain(t["norm1"], self.taps.wp, device, zero_centred=False)
        if self.mlp is not None:
            self.mlp.load(part("mlp."), device)
            self.g_post2 = norm_gain(t["norm2"], self.taps.wp, device, zero_centred=False)
        return t["dwa"]

    def stateful(self):
        return [self.taps, self.mixer] if isinstance(self.mixer, LinearAttention) else [self.taps]


class GulozenForCausalLM(nn.Module):

    def __init__(self, config):
        super().__init__()
        self.config = config
        self.dtype = config.torch_dtype
        self.layers = nn.ModuleList([GulozenLayer(config, s) for s in config.layers])
        self.residual = DepthResidual(config.hidden_size, len(config.layers), config.norm_groups, config.rms_norm_eps, self.dtype)
        self.embed = self.head = None

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
        self.residual.load(need("final.norm"), [layer.load_from(fetch, f"l{i}", dev) for i, layer in enumerate(self.layers)], dev)
        for m in self._attention:
            m.rot.prepare(dev)

    # ------------------------------------------------------------------ cache and state
    @property
    def _attention(self):
        return [layer.mixer for layer in self.layers if isinstance(layer.mixer, LatentAttention)]

    @property
    def windows(self) -> list[int]:
        return sorted({m.window for m in self._attention})

    @property
    def tile_sizes(self) -> list[int]:
        return sorted({m.tokens_per_tile for m in self._attention})

    @property
    def max_short_portion(self) -> int:
        """Longest portion of a sequence that takes the kernels for few rows (all of them in fp32, or with heads beyond the expanded
        attention's sizes)."""
        att = self._attention
        if self.dtype != torch.bfloat16 or not all(m.can_expand for m in att):
            return 1 << 30
        return max([m.break_even for m in att], default=MAX_SHORT)

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
    def _mix(self, layer, h, meta, tables):
        if isinstance(layer.mixer, LinearAttention):
            return layer.mixer(h, meta)
        return layer.mixer(h, meta, cs=layer.mixer.rot.shared_table(meta.pos, tables))

    def forward(self, meta, residual_tap: list | None = None) -> torch.Tensor:
        """fp32 logits [meta.want_rows, vocab] of the wanted rows of a step.  residual_tap (a list) receives what every layer hands on
        [T, width]."""
        cfg, res = self.config, self.residual
        planes = res.planes(meta.ids.numel(), meta.ids.device)
        hip_ops.embed_rows(meta.ids, self.embed, cfg.padded_width, scale=cfg.embedding_scale, out=planes[0])
        tables: dict = {}
        x, h = res.first(planes, self.layers[0].taps, meta)
        for i, layer in enumerate(self.layers):
            y, g_post = self._mix(layer, h, meta, tables), layer.g_post1
            if layer.mlp is not None:
                x, rows = res.inside(x, y, g_post)
                y, g_post = layer.mlp(rows), layer.g_post2
            if residual_tap is not None:
                residual_tap.append(res.result(i, planes, x, y, g_post)[:, : cfg.hidden_size])
            if i + 1 < len(self.layers):
                x, h = res.behind(i, planes, x, y, g_post, self.layers[i + 1].taps, meta)
        if meta.want.numel() == 0:
            return torch.empty((0, cfg.vocab_size), dtype=torch.float32, device=x.device)
        return hip_ops.linear_act(res.last(planes, x, y, g_post, meta.want), self.head, out_f32=True)[:, : cfg.vocab_size]
