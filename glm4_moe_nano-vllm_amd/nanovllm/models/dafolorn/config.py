"""Configuration of the Dafolorn design: config.json -> the namespace the engine and the model read.  Every size and
constant comes from the file; unknown mixers, feed-forwards or masks are refused rather than guessed."""
from __future__ import annotations

import types

import torch

from nanovllm.hip_ops import round8
from nanovllm.models.layer_loop import layer_runs, read_loop  # noqa: F401

MAX_POSITIONS = 1 << 30  # attention has no positional term: nothing limits a sequence but memory


class LayerSpec(types.SimpleNamespace):
    """One entry of `layers`: mixer type and sizes, feed-forward kind and sizes (ff None: no feed-forward)."""


def _layer(i: int, e: dict) -> LayerSpec:
    if e["type"] != "latent_attention":
        raise NotImplementedError(f"layer {i}: mixer {e['type']!r}")
    m = e["mixer"]
    window = int(m["mask"]["size"])
    s = LayerSpec(index=i, type=e["type"], heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), kv_rank=int(m["kv_rank"]),
                  scale=float(m["scale"]), window=window, mlp=None, ff=0)
    mlp = e.get("mlp")
    if mlp is not None:
        if mlp["kind"] != "dense":
            raise NotImplementedError(f"layer {i}: feed-forward {mlp['kind']!r}")
        s.mlp, s.ff = mlp["kind"], int(mlp["ff"])
    if min(s.heads, s.dim, s.vdim, s.kv_rank, window) < 1:
        raise ValueError(f"layer {i}: sizes must be positive")
    return s


def read_config(raw: dict) -> types.SimpleNamespace:
    d = raw if isinstance(raw, dict) else dict(vars(raw))
    layers = [_layer(i, e) for i, e in enumerate(d["layers"])]
    loop = read_loop(d.get("loop"), len(layers))
    cap = d.get("logit_softcap")
    return types.SimpleNamespace(
        raw=d, model_type="dafolorn", vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), padded_width=round8(int(d["width"])),
        layers=layers, loop=loop, rms_norm_eps=float(d["norm"]["eps"]), conv_taps=int(d["canon"]["taps"]),
        logit_softcap=None if cap is None else float(cap), num_hidden_layers=len(layers), max_position_embeddings=MAX_POSITIONS,
        max_window=max(s.window for s in layers), torch_dtype=torch.bfloat16)
