"""Greedy generation from token ids on the command line, for any registered model.

    bin/generate --model DIR --prompt-ids 1,2,3 --prompt-ids 7,8 --max-tokens 16

Prints one JSON line per prompt: {"prompt": [...], "completion": [...]}."""
import argparse
import json
import sys

import torch

from .engine.llm_engine import LLMEngine
from .models import load_config


def main(argv=None):
    ap = argparse.ArgumentParser(prog="generate", description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    ap.add_argument("--model", required=True, help="folder with config.json and *.safetensors")
    ap.add_argument("--prompt-ids", action="append", required=True, help="comma-separated token ids; repeat for a batch")
    ap.add_argument("--max-tokens", type=int, default=16)
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"], help="float32: models that run in true 32-bit only")
    ap.add_argument("--random-weights", action="store_true", help="random weights of the configuration instead of the checkpoint")
    ap.add_argument("--max-model-len", type=int, default=4096)
    ap.add_argument("--max-num-seqs", type=int, default=32)
    ap.add_argument("--max-num-batched-tokens", type=int, default=16384)
    ap.add_argument("--kvcache-tokens", type=int, default=0, help="tokens the cache pool holds (0: enough for the batch)")
    ap.add_argument("--enforce-eager", action="store_true", help="no HIP-graph decode sessions")
    a = ap.parse_args(argv)
    prompts = [[int(t) for t in p.split(",")] for p in a.prompt_ids]
    cfg = load_config(a.model)
    if hasattr(cfg, "dtype"):
        cfg.dtype = getattr(torch, a.dtype)
    elif a.dtype != "bfloat16":
        ap.error(f"{cfg.name} runs in bfloat16 only")
    bs = cfg.kvcache_block_size
    blocks = -(-a.kvcache_tokens // bs) or sum(-(-(len(p) + a.max_tokens) // bs) for p in prompts)
    longest = min(a.max_model_len, getattr(cfg, "max_position_embeddings", a.max_model_len))
    engine = LLMEngine(cfg, blocks, weights=None if a.random_weights else a.model, max_model_len=longest, max_num_seqs=a.max_num_seqs,
                       max_num_batched_tokens=a.max_num_batched_tokens, enforce_eager=a.enforce_eager)
    for p, c in zip(prompts, engine.generate(prompts, a.max_tokens)):
        print(json.dumps({"prompt": p, "completion": c}))
    return 0


if __name__ == "__main__":
    sys.exit(main())
