"""Replays given token ids through the engine step by step and hands out logits; nothing is sampled.

``TraceReplayer`` drives the engine's own scheduler state (blocks and state slots) and runner; a step
is one batch of spans, portions of some requests beside single tokens of others.  ``main`` is the
command line around it: steps arrive as JSON lines on standard input, logits go to files.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
from typing import Dict, List, Optional

import torch

from . import registry
from .config import EngineConfig
from .model_runner import ModelRunner, Span
from .scheduler import Scheduler
from .sequence import Sequence

LIVE_REQUESTS = 4                # state slots; requests that may be live at the same time
COUNT_UNIT = 64                  # the caller rounds every live request up to a multiple of this


class TraceReplayer:

    def __init__(self, model_dir: str, dtype: str = "bfloat16", max_tokens: int = 4096, enforce_eager: bool = False):
        cfg = registry.load_config(model_dir)
        if not cfg.portions:
            raise NotImplementedError(f"{cfg.name} does not take portions of prompts")
        block = Sequence.block_size
        # a request may reach into one more block than its count, rounded up by the caller, says
        blocks = (max_tokens + LIVE_REQUESTS * (block - COUNT_UNIT)) // block
        config = EngineConfig(model_dir, dtype=dtype, max_num_seqs=LIVE_REQUESTS, max_model_len=max_tokens,
                              max_num_batched_tokens=max(max_tokens, LIVE_REQUESTS), num_kvcache_blocks=max(blocks, 1),
                              enforce_eager=enforce_eager)
        self.scheduler = Scheduler(config)
        self.runner = ModelRunner(config)
        self.live: Dict[str, Sequence] = {}

    def step(self, entries: List[dict], end: List[str]) -> Optional[torch.Tensor]:
        """Runs the next tokens of every entry as one batch; fp32 logits ``[wanted, vocab]`` on the host."""
        spans = []
        for e in entries:
            tokens = e["tokens"]
            if not tokens:
                continue
            seq = self.live.get(e["id"])
            if seq is None:
                seq = self.live[e["id"]] = Sequence(tokens)
            else:
                seq.token_ids.extend(tokens)
            self.scheduler.hold(seq)
            spans.append(Span(seq, len(seq) - len(tokens), len(tokens), list(e.get("want", []))))
        logits = self.runner.run_spans(spans) if spans else None
        out = None if logits is None else logits.float().cpu()
        torch.cuda.synchronize()
        for name in end:
            if name in self.live:
                self.scheduler.release(self.live.pop(name))
        return out


def main(argv=None, before_loading=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="Feeds token ids through a model step by step and writes logits. "
                                 "Reads one JSON object a line: {\"step\", \"entries\": [{\"id\", \"tokens\", \"want\"}], \"end\": [ids]}.")
    ap.add_argument("--model", required=True, help="folder with config.json and *.safetensors")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--out", required=True, help="folder that receives <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold at any time")
    args = ap.parse_args(argv)
    if args.dtype not in registry.load_config(args.model).dtypes:
        print(f"this model does not run in {args.dtype}", file=sys.stderr)
        return 3
    if before_loading is not None:
        before_loading(args.model)
    replayer = TraceReplayer(args.model, args.dtype, args.max_tokens)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = replayer.step(step["entries"], step.get("end", []))
        if logits is not None:
            part = os.path.join(args.out, f".{step['step']}.part")
            logits.numpy().astype("<f4").tofile(part)
            os.replace(part, os.path.join(args.out, f"{step['step']}.f32"))
        print(f"done {step['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
