"""A group of layers that runs several times in a row with the same weights, every pass with its own cache and state."""
from __future__ import annotations

import types


def read_loop(loop: dict | None, layers: int):
    """config `loop` {start, stop, times} -> namespace, or None: no layer runs twice."""
    if loop is None:
        return None
    loop = types.SimpleNamespace(start=int(loop["start"]), stop=int(loop["stop"]), times=int(loop["times"]))
    if not 0 <= loop.start < loop.stop <= layers or loop.times < 1:
        raise ValueError(f"loop {vars(loop)} does not fit {layers} layers")
    return loop


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


def run_indices(cfg) -> tuple[list, list]:
    """(which run of its layer every entry of layer_runs is, runs per layer)."""
    count, index = [0] * len(cfg.layers), []
    for i, _ in layer_runs(cfg):
        index.append(count[i])
        count[i] += 1
    return index, count
