"""Token-id generation from a checkpoint directory of any causal language model of the registry (cogstream_amd.auto):

    python -m cogstream_amd.generate --model_path DIR --prompt 5,17,3 [--prompt 8,1 ...] [--max_new_tokens N] [--greedy]

Prompts (comma-separated ids; without --prompt one JSON list a line on standard input) run as one batch; one JSON line per
prompt comes back, in order: {"prompt": index, "tokens": [new ids]}."""
from __future__ import annotations

import argparse
import json
import sys


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(description="Generate token ids from token-id prompts.")
    ap.add_argument("--model_path", required=True, help="Path to the model directory.")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--prompt", action="append", help="token ids with commas between them; repeat for more prompts")
    ap.add_argument("--max_new_tokens", type=int, default=64)
    ap.add_argument("--max_batch", type=int, default=64, help="requests that run at once")
    ap.add_argument("--greedy", action="store_true", help="no sampling, whatever the checkpoint's generation config says")
    ap.add_argument("--temperature", type=float, help="sample at this temperature")
    ap.add_argument("--top_k", type=int)
    ap.add_argument("--top_p", type=float)
    ap.add_argument("--repetition_penalty", type=float)
    ap.add_argument("--seed", type=int, default=0)
    ap.add_argument("--eos", type=int, action="append", help="end token; repeat for more")
    args = ap.parse_args(argv)
    import torch

    from .auto import AutoModelForCausalLM
    prompts = ([[int(t) for t in p.split(",")] for p in args.prompt] if args.prompt
               else [json.loads(line) for line in sys.stdin if line.strip()])
    if not prompts:
        ap.error("no prompts")
    model = AutoModelForCausalLM.from_pretrained(args.model_path, torch_dtype=getattr(torch, args.dtype))
    opts = {k: v for k, v in model.generation_config.items() if k in ("do_sample", "temperature", "top_k", "top_p", "repetition_penalty",
                                                                      "eos_token_id")}
    opts.update({k: getattr(args, k) for k in ("temperature", "top_k", "top_p", "repetition_penalty") if getattr(args, k) is not None})
    if args.eos:
        opts["eos_token_id"] = args.eos
    if isinstance(opts.get("eos_token_id"), int):
        opts["eos_token_id"] = [opts["eos_token_id"]]
    if args.greedy:
        opts["do_sample"] = False
    elif args.temperature is not None:
        opts["do_sample"] = True
    with torch.inference_mode():
        out = model.llm.generate_batch(prompts, max_new_tokens=args.max_new_tokens, max_batch=args.max_batch, seed=args.seed, **opts)
    for i, toks in enumerate(out):
        sys.stdout.write(json.dumps({"prompt": i, "tokens": toks}) + "\n")
    return 0


if __name__ == "__main__":
    raise SystemExit(main())
