"""Replay of a token trace: given tokens are fed step by step through an engine and logits are written out; nothing is sampled.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N  < steps.jsonl

Every input line is one step: {"step": n, "entries": [{"id": ..., "tokens": [...], "want": [places]}], "end": [ids]}.  All entries of a step are one
batch.  The logits at the wanted places go to DIR/<n>.f32 (little-endian fp32 rows, in order), then the line "done <n>" is printed.  `end` lists
requests whose cache pages and state slots are given back after the step.  The cache holds N tokens, and there are four state slots."""
import argparse
import json
import os
import sys

import torch

from .engine.llm_engine import LLMEngine
from .models import load_config

LIVE_REQUESTS = 4


class TraceRunner:
    def __init__(self, model, dtype, max_tokens):
        block = 64
        cfg = load_config(model, dtype=dtype, max_position_embeddings=max(max_tokens, 1), kvcache_block_size=block)
        # the pool is for all live requests; one of them may have fewer positions (a learned table is as long as it is)
        self.engine = LLMEngine(cfg, num_kvcache_blocks=-(-max_tokens // block), weights=model, max_num_seqs=LIVE_REQUESTS,
                                max_model_len=min(max_tokens, cfg.max_position_embeddings))
        if not self.engine.runner.mixed_batches:
            raise SystemExit(f"{self.engine.cfg.name}: trace replay needs a model that takes mixed batches")
        self.live = {}

    def step(self, entries, end):
        portions = []
        for e in entries:
            seq = self.live.get(e["id"])
            if seq is None:
                seq = self.live[e["id"]] = self.engine.sequence(e["tokens"])
            else:
                for t in e["tokens"]:
                    seq.append_token(t)
            portions.append((seq, len(e["tokens"])))
        logits = self.engine.feed(portions, [e["want"] for e in entries]) if portions else None
        out = None if logits is None else logits.float().cpu().contiguous()
        for i in end:
            self.engine.release(self.live.pop(i))
        return out


def main(argv=None, prepare=None):
    """prepare(model folder): called before anything is loaded (compiles what is missing)."""
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    ap.add_argument("--model", required=True)
    ap.add_argument("--dtype", required=True, choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True)
    ap.add_argument("--max-tokens", required=True, type=int)
    a = ap.parse_args(argv)
    if prepare is not None:
        prepare(a.model)
    runner = TraceRunner(a.model, getattr(torch, a.dtype), a.max_tokens)
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = runner.step(s["entries"], s["end"])
        if logits is not None:
            with open(os.path.join(a.out, f"{s['step']}.f32"), "wb") as f:
                f.write(logits.numpy().astype("<f4").tobytes())
        print(f"done {s['step']}", flush=True)
    return 0
