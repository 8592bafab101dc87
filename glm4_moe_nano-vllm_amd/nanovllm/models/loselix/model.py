"""Loselix: a decoder with one norm per layer, whose mixer and feed-forward (square of relu, where a layer has one) both read it and are
added to a 32-bit residual; mixers are attention of three kinds — differential with a soft cap, softmax with a gate per head, sigmoid
weights over keys that are the values — and a group of layers runs several times with the same weights, the embedding being added again
ahead of every pass but the first.

The model runs StepBatch inputs (engine/step_batch.py): any mixture of prompt portions and decoded tokens.  Every layer run (a looped
layer once per pass) has its own cache; there is no other state."""
from __future__ import annotations

import torch
import torch.nn as nn

from nanovllm import hip_ops
from nanovllm.layers.group_attention import GroupAttention
from nanovllm.layers.parallel_block import ParallelBlock
from nanovllm.layers.rotary_embedding import HalfRotary
from nanovllm.layers.seq_norm import norm_gain
from nanovllm.models.layer_loop import layer_runs, run_indices
from nanovllm.utils.loader import load_prefixed

MAX_SHORT = 16          # longest portion that takes the kernels for few rows per sequence


def make_mixer(cfg, s, runs: int) -> GroupAttention:
    kinds = {"attention": lambda: dict(rot=HalfRotary(s.dim, s.rot_dims, s.rot_base), cap=s.softcap, diff=s.diff),
             "attention_2": lambda: dict(rot=HalfRotary(s.dim, s.rot_dims, s.rot_base), gate="head"),
             "attention_3": lambda: dict(sigmoid_kv=True, temperature=(s.temp_coef, s.temp_every), gate="column")}
    return GroupAttention(cfg.hidden_size, s.heads, s.kv_heads, s.dim, s.vdim, s.scale, cfg.torch_dtype, joint=True, runs=runs, eps=cfg.rms_norm_eps, **kinds[s.type]())


class LoselixLayer(nn.Module):

    def __init__(self, cfg, spec, runs: int):
        super().__init__()
        self.spec = spec
        self.block = ParallelBlock(cfg.hidden_size, make_mixer(cfg, spec, runs), spec.ff, cfg.torch_dtype)
        self.g = None

    @property
    def mixer(self) -> GroupAttention:
        return self.block.mixer

    def load_from(self, fetch, prefix: str, device) -> None:
        t = {k[len(prefix) + 1:]: v for k, v in fetch(prefix).items()}
        if not t:
            raise ValueError(f"no tensors under '{prefix}'")
        part = lambda p: {k[len(p):]: v for k, v in t.items() if k.startswith(p)}  # noqa: E731
        self.g = norm_gain(t["norm1"], self.block.wp, device, zero_centred=False)
        self.block.load(part("mix."), part("mlp."), device)


class LoselixForCausalLM(nn.Module):

    def __init__(self, config):
        super().__init__()
        self.config = config
        self.dtype = config.torch_dtype
        self.runs = layer_runs(config)
        self.run_index, count = run_indices(config)
        self.layers = nn.ModuleList([LoselixLayer(config, s, count[s.index]) for s in config.layers])
        self.embed = self.head = self.g_final = None

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
        self.g_final = norm_gain(need("final.norm"), wp, dev, zero_centred=False)
        for i, layer in enumerate(self.layers):
            layer.load_from(fetch, f"l{i}", dev)

    # ------------------------------------------------------------------ cache and state
    windows = ()            # no kernel of this model wants a step's history gathered

    @property
    def chunk_tiles(self) -> list[tuple]:
        return sorted({(layer.mixer.chunk, layer.mixer.tile_rows) for layer in self.layers})

    @property
    def tile_sizes(self) -> list[int]:
        return sorted({layer.mixer.tokens_per_tile for layer in self.layers})

    @property
    def max_short_portion(self) -> int:
        """Longest portion of a sequence that takes the kernels for few rows (all of them in fp32)."""
        return MAX_SHORT if self.dtype == torch.bfloat16 else 1 << 30

    def cache_bytes_per_token(self) -> int:
        return sum(layer.mixer.cache_bytes_per_token() for layer in self.layers)

    def state_bytes_per_slot(self) -> int:
        return 0

    def allocate(self, num_blocks: int, block_size: int, num_slots: int, device) -> None:
        for layer in self.layers:
            layer.mixer.allocate_cache(num_blocks, block_size, device)

    # ------------------------------------------------------------------ step
    def forward(self, meta, residual_tap: list | None = None) -> torch.Tensor:
        """fp32 logits [meta.want_rows, vocab] of the wanted rows of a step.  residual_tap (a list) receives the residual stream [T, width]
        after every layer run."""
        cfg, wp = self.config, self.config.padded_width
        tables: dict = {}

        def norm(x, y, **kw):
            return hip_ops.residual_norm(x, cfg.hidden_size, wp, cfg.rms_norm_eps, y=y, act_dtype=self.dtype, **kw)

        x = y = None
        for (i, first_of_pass), r in zip(self.runs, self.run_index):
            layer, rot = self.layers[i], self.layers[i].mixer.rot
            x, h = norm(x, y, g=layer.g, embed=(meta.ids, self.embed) if x is None or first_of_pass else None)
            y = layer.block(h, meta, r, rot.shared_table(meta.pos, tables) if rot is not None else None)
            if residual_tap is not None:
                residual_tap.append(norm(x, y)[0][:, : cfg.hidden_size])
        if meta.want.numel() == 0:
            return torch.empty((0, cfg.vocab_size), dtype=torch.float32, device=x.device)
        _, h = norm(x, y, g=self.g_final, rows=meta.want, keep_x=False)
        return hip_ops.linear_act(h, self.head, out_f32=True)[:, : cfg.vocab_size]
