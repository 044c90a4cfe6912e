"""bin/trace_run — replay a trace of token ids and write logits.

Reads steps from standard input, one JSON object a line:
  {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [1]}],
   "end": []}
and writes OUT/<step>.f32 (little-endian floats, [wanted, vocab]) for steps in
which logits are wanted; prints "done <step>" after every step.
"""
from __future__ import annotations

import argparse
import json
import os
import sys


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run",
                                 description=__doc__.split("\n")[0])
    ap.add_argument("--model", required=True, help="model folder")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"],
                    default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="tokens that live requests hold at any time")
    ap.add_argument("--max-requests", type=int, default=4,
                    help="requests that are live at any time")
    ap.add_argument("--device", default="cuda")
    ap.add_argument("--eager", action="store_true",
                    help="no hipGraph capture of decode steps")
    args = ap.parse_args(argv)

    with open(os.path.join(args.model, "config.json")) as f:
        arch = json.load(f).get("architecture")
    if args.device == "cuda":
        # compile what this family runs on, before anything imports it
        from ..utils import hip_build
        hip_build.ensure(*hip_build.EXTENSIONS_OF.get(arch, ("_hip_ops",)))
    from ..engine.trace import TraceSession
    from ..models.registry import load_config
    import torch
    if args.device == "cuda" and not torch.cuda.is_available():
        print("no GPU visible", file=sys.stderr)
        return 1
    model = load_config(args.model)
    model.dtype = args.dtype
    session = TraceSession(model, args.max_tokens,
                           max_requests=args.max_requests, device=args.device,
                           enforce_eager=args.eager or args.device != "cuda")
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = session.step(step.get("entries", []), step.get("end", []))
        if logits.shape[0]:
            path = os.path.join(args.out, f"{step['step']}.f32")
            with open(path, "wb") as f:
                f.write(logits.contiguous().numpy().astype("<f4").tobytes())
        print(f"done {step['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
