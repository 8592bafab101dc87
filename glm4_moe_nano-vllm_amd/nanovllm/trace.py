"""Replay of a token trace: given token ids go through the engine step by step and the logits that are asked for are written
out.  Nothing is sampled.  The engine's own scheduler primitives (cache blocks, state slots), step function and kernels run the
steps; this module only reads the steps and writes the results.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N  < steps.jsonl

A step is one JSON object a line: {"step": n, "entries": [{"id": ..., "tokens": [...], "want": [places]}], "end": [ids]}.
Logits of a step's wanted places go to DIR/<step>.f32 (little-endian fp32, [wanted, vocab], in the order of the entries);
`done <step>` is printed after every step.  Exit code 3: the model does not run in the given dtype."""
from __future__ import annotations

import argparse
import json
import os
import sys

MAX_LIVE = 4       # requests that may hold cache and state at a time
UNIT = 64          # --max-tokens counts every request rounded up to a multiple of this


class TraceSession:
    """Requests by name on top of an engine that runs step batches."""

    def __init__(self, model: str, dtype: str, max_tokens: int, enforce_eager: bool = False):
        from nanovllm.engine.llm_engine import LLMEngine
        blocks = -(-max_tokens // UNIT)
        self.engine = LLMEngine(model, dtype=dtype, kvcache_block_size=UNIT, num_kvcache_blocks=blocks, max_num_seqs=MAX_LIVE,
                                max_model_len=blocks * UNIT, max_num_batched_tokens=blocks * UNIT, enforce_eager=enforce_eager)
        self.scheduler = self.engine.scheduler
        self.live: dict = {}

    def step(self, entries: list[dict], end: list):
        """Runs one batch; returns the wanted logits as a CPU fp32 tensor, or None."""
        from nanovllm.engine.sequence import Sequence
        batch = []
        for e in entries:
            if not e["tokens"]:
                continue
            seq = self.live.get(e["id"])
            if seq is None:
                seq = self.live[e["id"]] = Sequence(e["tokens"])
            else:
                for t in e["tokens"]:
                    seq.append_token(t)
            batch.append((seq, self.scheduler.feed(seq, len(e["tokens"]), e.get("want", []))))
        out = None
        if batch:
            logits = self.engine.model_runner.call("step_logits", [c for _, c in batch])
            if any(c.want for _, c in batch):
                out = logits.cpu()
        for seq, chunk in batch:
            self.scheduler.advance(seq, len(chunk.tokens))
        for name in end:
            seq = self.live.pop(name, None)
            if seq is not None:
                self.scheduler.release(seq)
        return out

    def close(self):
        self.engine.exit()


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="replay a token trace and write logits")
    ap.add_argument("--model", required=True)
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True)
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens live requests hold at a time, each rounded up to a multiple of 64")
    ap.add_argument("--eager", action="store_true", help="no HIP graphs")
    a = ap.parse_args(argv)
    from nanovllm.models.registry import find_model
    with open(os.path.join(a.model, "config.json")) as f:
        entry = find_model(json.load(f))
    if a.dtype not in entry.dtypes:
        print(f"{entry.name} does not run in {a.dtype}", file=sys.stderr)
        return 3
    if not entry.step_batches:
        print(f"{entry.name} does not run step batches", file=sys.stderr)
        return 2
    session = TraceSession(a.model, a.dtype, a.max_tokens, a.eager)
    os.makedirs(a.out, exist_ok=True)
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = session.step(s.get("entries", []), s.get("end", []))
        if logits is not None:
            with open(os.path.join(a.out, f"{s['step']}.f32"), "wb") as f:
                f.write(logits.contiguous().numpy().astype("<f4").tobytes())
        print(f"done {s['step']}", flush=True)
    session.close()
    return 0


if __name__ == "__main__":
    sys.exit(main())
