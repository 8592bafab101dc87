"""Generation from the command line:

    python -m nanovllm --model DIR [--prompt TEXT | --prompt-ids 1,2,3] ... [--max-tokens 64] [--temperature 0] [--dtype float32]

The model class follows from DIR/config.json (models/registry.py).  Models without a tokenizer take --prompt-ids."""
from __future__ import annotations

import argparse
import json
import sys


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="python -m nanovllm")
    ap.add_argument("--model", required=True)
    ap.add_argument("--prompt", action="append", default=[])
    ap.add_argument("--prompt-ids", action="append", default=[], help="comma-separated token ids; may be given several times")
    ap.add_argument("--max-tokens", type=int, default=64)
    ap.add_argument("--temperature", type=float, default=0.0)
    ap.add_argument("--ignore-eos", action="store_true")
    ap.add_argument("--dtype", default=None)
    ap.add_argument("--max-model-len", type=int, default=4096)
    ap.add_argument("--max-num-seqs", type=int, default=64)
    ap.add_argument("--tensor-parallel-size", type=int, default=1)
    ap.add_argument("--enforce-eager", action="store_true")
    a = ap.parse_args(argv)
    prompts = a.prompt + [[int(t) for t in p.split(",")] for p in a.prompt_ids]
    if not prompts:
        ap.error("no prompt")
    from nanovllm import LLM, SamplingParams
    llm = LLM(a.model, dtype=a.dtype, max_model_len=a.max_model_len, max_num_seqs=a.max_num_seqs, enforce_eager=a.enforce_eager,
              tensor_parallel_size=a.tensor_parallel_size)
    out = llm.generate(prompts, SamplingParams(temperature=a.temperature, max_tokens=a.max_tokens, ignore_eos=a.ignore_eos), use_tqdm=False)
    for o in out:
        print(json.dumps(o))
    llm.exit()
    return 0


if __name__ == "__main__":
    sys.exit(main())
