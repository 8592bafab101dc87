"""Configuration of the Napadra design: config.json -> the namespace the engine and the model read.  Every size and constant
comes from the file; unknown mixers, feed-forwards or masks are refused rather than guessed."""
from __future__ import annotations

import types

import torch

from nanovllm.engine.key_reach import KeyReach
from nanovllm.hip_ops import round8

MAX_POSITIONS = 1 << 30  # sinusoids and chunks go on for ever: nothing limits a sequence but memory


class LayerSpec(types.SimpleNamespace):
    """One entry of `layers`: mixer type and sizes, feed-forward kind and sizes (mlp None: no feed-forward)."""


def _layer(i: int, e: dict, earlier: list) -> LayerSpec:
    m = e["mixer"]
    s = LayerSpec(index=i, type=e["type"], heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), mlp=None, ff=0, limit=0.0)
    if s.type == "attention":
        s.kv_heads, s.scale, s.kv_from = int(m["kv_heads"]), float(m["scale"]), m.get("kv_from")
        unknown = set(m["mask"]) - {"size"}
        if unknown:
            raise NotImplementedError(f"layer {i}: mask with {sorted(unknown)}")
        s.chunk = int(m["mask"]["size"])
        if s.kv_heads < 1 or s.heads % s.kv_heads or s.chunk < 1:
            raise ValueError(f"layer {i}: {s.heads} heads over {s.kv_heads} key/value heads, chunks of {s.chunk}")
        if s.kv_from is not None:
            s.kv_from = int(s.kv_from)
            j = earlier[s.kv_from] if 0 <= s.kv_from < i else None
            if j is None or j.type != "attention" or j.kv_from is not None or (j.kv_heads, j.dim, j.vdim) != (s.kv_heads, s.dim, s.vdim):
                raise ValueError(f"layer {i}: no keys and values of its shape in layer {s.kv_from}")
    elif s.type == "mlstm":
        s.gate_cap = float(m["gate_cap"])
        if s.gate_cap <= 0:
            raise ValueError(f"layer {i}: a gate cap of {s.gate_cap}")
    else:
        raise NotImplementedError(f"layer {i}: mixer {s.type!r}")
    mlp = e.get("mlp")
    if mlp is not None:
        if mlp["kind"] != "dense":
            raise NotImplementedError(f"layer {i}: feed-forward {mlp['kind']!r}")
        s.mlp, s.ff, s.limit = mlp["kind"], int(mlp["ff"]), float(mlp["limit"])
    if min(s.heads, s.dim, s.vdim) < 1 or (s.mlp is not None and s.ff < 1):
        raise ValueError(f"layer {i}: sizes must be positive")
    return s


def read_config(raw: dict) -> types.SimpleNamespace:
    d = raw if isinstance(raw, dict) else dict(vars(raw))
    layers: list = []
    for i, e in enumerate(d["layers"]):
        layers.append(_layer(i, e, layers))
    streams = int(d["streams"])
    if streams < 1:
        raise ValueError(f"{streams} streams")
    return types.SimpleNamespace(
        raw=d, model_type="napadra", vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), padded_width=round8(int(d["width"])), layers=layers,
        streams=streams, residual_mult=float(d["residual_mult"]), rms_norm_eps=float(d["norm"]["eps"]), num_hidden_layers=len(layers),
        max_position_embeddings=MAX_POSITIONS, key_reach=KeyReach(chunks=tuple(sorted({s.chunk for s in layers if s.type == "attention"}))),
        torch_dtype=torch.bfloat16)
