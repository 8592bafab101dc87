"""Dafolorn: a decoder with a 32-bit residual stream, norms in front of and behind every sublayer, a short causal convolution
on what each sublayer reads, windowed latent attention with sinks, an ungated xIELU feed-forward, and a group of layers that
runs several times with the same weights, the embedding output being mixed back in ahead of every pass.

The model runs StepBatch inputs (engine/step_batch.py): any mixture of prompt portions and decoded tokens.  Every layer run
(a looped layer once per pass) has its own latent cache and convolution state."""
from __future__ import annotations

import torch
import torch.nn as nn

from nanovllm import hip_ops
from nanovllm.layers.dense_mlp import DenseMLP
from nanovllm.layers.latent_attention import LatentAttention
from nanovllm.layers.linear import PaddedLinear
from nanovllm.layers.seq_norm import SublayerEntry, norm_gain
from nanovllm.models.layer_loop import layer_runs, run_indices
from nanovllm.utils.loader import load_prefixed


class DafolornLayer(nn.Module):

    def __init__(self, cfg, spec, runs: int):
        super().__init__()
        self.spec, dt = spec, cfg.torch_dtype
        self.entry1 = SublayerEntry(cfg.hidden_size, cfg.conv_taps, cfg.rms_norm_eps, runs)
        self.mixer = LatentAttention(cfg.hidden_size, spec.heads, spec.dim, spec.vdim, spec.kv_rank, spec.window, spec.scale,
                                     cfg.rms_norm_eps, dt, runs)
        self.entry2 = self.mlp = None
        if spec.mlp is not None:
            self.entry2 = SublayerEntry(cfg.hidden_size, cfg.conv_taps, cfg.rms_norm_eps, runs)
            self.mlp = DenseMLP(cfg.hidden_size, spec.ff, dt)
        self.g_post1 = self.g_post2 = None

    def load_from(self, fetch, prefix: str, device) -> None:
        t = {k[len(prefix) + 1:]: v for k, v in fetch(prefix).items()}
        if not t:
            raise ValueError(f"no tensors under '{prefix}'")
        wp = self.entry1.wp
        sub = lambda p: {k[len(p):]: v for k, v in t.items() if k.startswith(p)}  # noqa: E731
        self.entry1.load(t["norm1"], t["canon1"], device)
        self.g_post1 = norm_gain(t["norm1b"], wp, device)
        self.mixer.load(sub("mix."), device)
        if self.mlp is not None:
            self.entry2.load(t["norm2"], t["canon2"], device)
            self.g_post2 = norm_gain(t["norm2b"], wp, device)
            self.mlp.load(sub("mlp."), device)

    def entries(self):
        return [e for e in (self.entry1, self.entry2) if e is not None]


class DafolornForCausalLM(nn.Module):

    def __init__(self, config):
        super().__init__()
        self.config = config
        self.dtype = config.torch_dtype
        self.runs = layer_runs(config)
        self.run_index, count = run_indices(config)
        self.layers = nn.ModuleList([DafolornLayer(config, s, count[s.index]) for s in config.layers])
        w = config.hidden_size
        self.loop_in = PaddedLinear([w, w], [config.padded_width], self.dtype) if config.loop else None
        self.embed = self.loop_step = self.g_final = None

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

        table = hip_ops.padded_weight(hip_ops.round8(V), wp, dtype=self.dtype, device=dev)
        table.zero_()
        table[:V, :w] = need("embed").to(device=dev, dtype=self.dtype)
        self.embed = table           # also the output projection
        self.g_final = norm_gain(need("final.norm"), wp, dev)
        if self.loop_in is not None:
            self.loop_in.load([need("loop.in")], dev)
            step = torch.zeros(cfg.loop.times, wp, dtype=self.dtype, device=dev)
            step[:, :w] = need("loop.step").to(device=dev, dtype=self.dtype)
            self.loop_step = step
        for i, layer in enumerate(self.layers):
            layer.load_from(fetch, f"l{i}", dev)

    # ------------------------------------------------------------------ cache and state
    @property
    def windows(self) -> list[int]:
        return sorted({s.window for s in self.config.layers})

    @property
    def tile_sizes(self) -> list[int]:
        return sorted({layer.mixer.tokens_per_tile for layer in self.layers})

    @property
    def max_short_portion(self) -> int:
        """Longest portion of a sequence that attends in the absorbed form."""
        if all(layer.mixer.can_expand for layer in self.layers):
            return max(layer.mixer.break_even for layer in self.layers)
        return 1 << 30

    def cache_bytes_per_token(self) -> int:
        return sum(layer.mixer.cache_bytes_per_token() for layer in self.layers)

    def state_bytes_per_slot(self) -> int:
        return 2 * sum(e.state_bytes() for layer in self.layers for e in layer.entries())

    def allocate(self, num_blocks: int, block_size: int, num_slots: int, device) -> None:
        for layer in self.layers:
            layer.mixer.allocate_cache(num_blocks, block_size, device)
            for e in layer.entries():
                e.allocate_state(2 * num_slots, device)

    # ------------------------------------------------------------------ step
    def forward(self, meta, residual_tap: list | None = None) -> torch.Tensor:
        """fp32 logits [meta.want_rows, vocab] of the wanted rows of a step.  residual_tap (a list) receives the residual
        stream [T, width] after every layer run."""
        cfg, dt = self.config, self.dtype
        T, wp, eps = meta.ids.numel(), cfg.padded_width, cfg.rms_norm_eps
        cat = torch.empty((T, 2 * wp), dtype=dt, device=meta.ids.device) if cfg.loop else None
        x = hip_ops.embed_rows(meta.ids, self.embed, wp, cat[:, wp:] if cat is not None else None)
        y = g_post = None            # output of the sublayer that is not yet in x, and its closing norm

        def tap(x):
            if residual_tap is not None and y is not None:
                residual_tap.append(x[:, : cfg.hidden_size].clone())

        for (i, first_of_pass), r in zip(self.runs, self.run_index):
            layer = self.layers[i]
            if first_of_pass is not None:
                x, _ = hip_ops.seq_norm(x, cfg.hidden_size, eps, y=y, g_post=g_post, act_dtype=dt, x_cast=cat[:, :wp],
                                        keep_x=residual_tap is not None)
                tap(x)
                x, y = self.loop_in(cat, bias=self.loop_step[first_of_pass], out_f32=True), None
            x, h = layer.entry1(x, y, g_post, meta, r, dt)
            tap(x)
            y, g_post = layer.mixer(h, meta, r), layer.g_post1
            if layer.mlp is not None:
                x, h = layer.entry2(x, y, g_post, meta, r, dt)
                y, g_post = layer.mlp(h), layer.g_post2
        if residual_tap is not None:
            tap(hip_ops.seq_norm(x, cfg.hidden_size, eps, y=y, g_post=g_post, act_dtype=dt)[0])
        if meta.want.numel() == 0:
            return torch.empty((0, cfg.vocab_size), dtype=torch.float32, device=x.device)
        _, h = hip_ops.seq_norm(x, cfg.hidden_size, eps, y=y, g_post=g_post, g_pre=self.g_final, rows=meta.want, act_dtype=dt, keep_x=False)
        act = hip_ops.NO_ACT if cfg.logit_softcap is None else (hip_ops.ACT_SOFTCAP, cfg.logit_softcap, 0.0)
        return hip_ops.linear_act(h, self.embed, act=act, out_f32=True)[:, : cfg.vocab_size]
