"""Command line of the engine: prompts of token ids in, generated token ids out, one JSON line each.

    bin/generate --model DIR --prompt 5,17,3 --prompt 9 --max-tokens 32 --temperature 0
    bin/generate --model DIR < prompts.jsonl            (one JSON list of token ids a line)
"""
from __future__ import annotations

import argparse
import json
import sys


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="generate", description="Generates from prompts of token ids with a model of the framework.")
    ap.add_argument("--model", required=True, help="folder with config.json and, where the family loads weights, *.safetensors")
    ap.add_argument("--prompt", action="append", help="comma-separated token ids; may be given several times (default: JSON lists on stdin)")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--max-tokens", type=int, default=64)
    ap.add_argument("--temperature", type=float, default=0.0, help="0: greedy")
    ap.add_argument("--max-model-len", type=int, default=4096)
    ap.add_argument("--max-num-seqs", type=int, default=64)
    ap.add_argument("--eos", type=int, default=-1, help="token id that ends a sequence")
    ap.add_argument("--seed", type=int, default=0)
    args = ap.parse_args(argv)
    if args.prompt:
        prompts = [[int(t) for t in p.split(",")] for p in args.prompt]
    else:
        prompts = [json.loads(line) for line in sys.stdin if line.strip()]
    from .llm import LLM
    from .sampling_params import SamplingParams
    llm = LLM(args.model, dtype=args.dtype, max_model_len=args.max_model_len, max_num_seqs=args.max_num_seqs, eos=args.eos, seed=args.seed)
    params = SamplingParams(temperature=args.temperature, max_tokens=args.max_tokens, ignore_eos=args.eos < 0)
    for prompt, out in zip(prompts, llm.generate(prompts, params)):
        print(json.dumps({"prompt": prompt, "token_ids": out["token_ids"]}), flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
