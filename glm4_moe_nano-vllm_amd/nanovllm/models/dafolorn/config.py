"""Configuration of the Dafolorn design: config.json -> the namespace the engine and the model read.  Every size and
constant comes from the file; unknown mixers, feed-forwards or masks are refused rather than guessed."""
from __future__ import annotations

import types

import torch

from nanovllm.hip_ops import round8

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
    loop = d.get("loop")
    if loop is not None:
        loop = types.SimpleNamespace(start=int(loop["start"]), stop=int(loop["stop"]), times=int(loop["times"]))
        if not 0 <= loop.start < loop.stop <= len(layers) or loop.times < 1:
            raise ValueError(f"loop {vars(loop)} does not fit {len(layers)} layers")
    cap = d.get("logit_softcap")
    return types.SimpleNamespace(
        raw=d, model_type="dafolorn", vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), padded_width=round8(int(d["width"])),
        layers=layers, loop=loop, rms_norm_eps=float(d["norm"]["eps"]), conv_taps=int(d["canon"]["taps"]),
        logit_softcap=None if cap is None else float(cap), num_hidden_layers=len(layers), max_position_embeddings=MAX_POSITIONS,
        max_window=max(s.window for s in layers), torch_dtype=torch.bfloat16)


def layer_runs(cfg) -> list:
    """The layers in the order they run: (layer index, pass number if this is the first layer of a pass else None)."""
    n = len(cfg.layers)
    if cfg.loop is None:
        return [(i, None) for i in range(n)]
    lo, hi = cfg.loop.start, cfg.loop.stop
    runs = [(i, None) for i in range(lo)]
    for t in range(cfg.loop.times):
        runs += [(i, t if i == lo else None) for i in range(lo, hi)]
    return runs + [(i, None) for i in range(hi, n)]
