"""bin/trace_run as a user calls it: a process of its own, steps on its standard input, logits in files."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from loselix_util import Reference, make_model, tokens

pytestmark = [pytest.mark.gpu, pytest.mark.timeout(120)]
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run(dtype, tmp_path):
    cfg, t = make_model(tmp_path / "m", "odd", 9)
    a, b = tokens(cfg, 150, 1), tokens(cfg, 40, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:100], "want": [0, 99]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[:2], "want": []}, {"id": "a", "tokens": a[100:101], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[101:102], "want": [0]}, {"id": "b", "tokens": b[2:], "want": [37, 1]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "b", "tokens": b, "want": [39]}], "end": []},
             {"step": 4, "entries": [{"id": "b", "tokens": b[:1], "want": []}, {"id": "a", "tokens": a[102:], "want": [47]}], "end": ["a", "b"]}]
    p = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", dtype, "--out",
                        str(tmp_path / "out"), "--max-tokens", "256"], input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True,
                       text=True, timeout=110)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [x for x in p.stdout.splitlines() if x.startswith("done")] == [f"done {i}" for i in range(5)]
    ref = {"a": Reference(cfg, t, a), "b": Reference(cfg, t, b)}
    want = {0: [("a", 0), ("a", 99)], 2: [("a", 101), ("b", 39), ("b", 3)], 3: [("b", 39)], 4: [("a", 149)]}
    assert sorted(os.listdir(tmp_path / "out")) == [f"{i}.f32" for i in want]
    for i, rows in want.items():
        got = torch.from_numpy(np.fromfile(tmp_path / "out" / f"{i}.f32", dtype="<f4")).view(-1, cfg["vocab"])
        assert got.shape[0] == len(rows)
        for g, (name, p) in zip(got, rows):
            ref[name].check_one(g, p, dtype)
