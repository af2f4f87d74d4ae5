"""Replays a trace of token steps through a model and writes the logits it asks for (bin/trace_run).

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR [--max-tokens N]

One JSON object a line on standard input:
    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}
entries are one batch: each request's next tokens, and the places among them whose logits are wanted; end: the requests that
are finished after the step. OUT/<step>.f32 holds the wanted logits in order, little-endian fp32 [wanted, vocab]; a line
"done <step>" follows every step."""
from __future__ import annotations

import argparse
import json
import os
import sys


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="Replay a trace of token steps and write the wanted logits.")
    ap.add_argument("--model", required=True, help="checkpoint directory (config.json, model.safetensors)")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--out", required=True, help="directory of the <step>.f32 files")
    ap.add_argument("--max-tokens", type=int, default=0, help="most tokens that live requests hold at any time (a hint; caches grow)")
    args = ap.parse_args(argv)
    import torch

    from .auto import AutoModelForCausalLM
    from .llm import Sequences
    model = AutoModelForCausalLM.from_pretrained(args.model, torch_dtype=getattr(torch, args.dtype))
    live = Sequences(model.llm)
    with torch.inference_mode():
        for line in sys.stdin:
            if not line.strip():
                continue
            rec = json.loads(line)
            logits = live.step([(e["id"], e["tokens"], e.get("want", [])) for e in rec["entries"]]) if rec.get("entries") else None
            if logits is not None:
                path = os.path.join(args.out, f"{rec['step']}.f32")
                with open(path + ".part", "wb") as f:
                    f.write(logits.contiguous().cpu().numpy().astype("<f4").tobytes())
                os.replace(path + ".part", path)
            else:
                torch.cuda.synchronize()
            for rid in rec.get("end", []):
                live.release(rid)
            sys.stdout.write(f"done {rec['step']}\n")
            sys.stdout.flush()
    return 0


if __name__ == "__main__":
    raise SystemExit(main())
