"""Command line: ``python -m onebit_amd <command>``.  The model class is chosen by the folder's config.json.

  generate   greedy continuation of token ids through the continuous batcher
  trace      replay a recorded schedule of steps (also: bin/trace_run)"""
from __future__ import annotations

import argparse
import json
import sys


def _trace_args(ap: argparse.ArgumentParser):
    ap.add_argument("--model", required=True, help="folder with config.json and the weights")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16",
                    help="bfloat16: the family's serving kernels; float32: everything in 32-bit (exit code 3 if the family has no such kernels)")
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, required=True, help="upper bound of the tokens held by all open requests together (sizes the cache)")


def trace_main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="replay a recorded schedule of steps through a model's serving engine and dump logits")
    _trace_args(ap)
    a = ap.parse_args(argv)
    from .trace import run
    return run(a.model, a.dtype, a.out, a.max_tokens)


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="onebit_amd", description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    sub = ap.add_subparsers(dest="command", required=True)
    _trace_args(sub.add_parser("trace", help="replay a trace from standard input"))
    g = sub.add_parser("generate", help="greedy generation")
    g.add_argument("--model", required=True)
    g.add_argument("--dtype", choices=["bfloat16", "float16", "float32"], help="default: the family's serving format")
    g.add_argument("--prompt", action="append", required=True, help="token ids, comma-separated; repeat for more requests")
    g.add_argument("--max-new-tokens", type=int, default=32)
    g.add_argument("--max-batch", type=int, default=32)
    g.add_argument("--prefill-chunk", type=int, help="prompt tokens of a request per step (default: whole prompts)")
    a = ap.parse_args(argv)
    if a.command == "trace":
        from .trace import run
        return run(a.model, a.dtype, a.out, a.max_tokens)
    import torch

    from .registry import load_model
    from .serving import ContinuousBatcher
    model = load_model(a.model, dtype=None if a.dtype is None else getattr(torch, a.dtype))
    prompts = [[int(t) for t in p.replace(",", " ").split()] for p in a.prompt]
    cb = ContinuousBatcher(model, max_batch=min(a.max_batch, max(len(prompts), 2)), max_len=max(len(p) for p in prompts) + a.max_new_tokens,
                           prefill_chunk=a.prefill_chunk)
    ids = [cb.add_request(p, a.max_new_tokens) for p in prompts]
    out = cb.run()
    for i in ids:
        print(json.dumps({"request": i, "tokens": out[i]}))
    return 0


if __name__ == "__main__":
    sys.exit(main())
