"""Replay a trace: run given token ids through a model step by step and write
logits. Nothing is sampled.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Each line of standard input is one step,

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [1]}],
     "end": ["b"]}

run as one batch by the StepRunner that also serves sessions. Requests are
admitted at their first entry and released when ``end`` names them. The
logits at the wanted places go to OUT/<step>.f32 (little-endian float32), and
``done <step>`` is printed after every step.
"""

from __future__ import annotations

import argparse
import json
import os
import sys
from typing import Dict, List, Optional

SLOTS = 4            # live requests
BLOCK = 64           # tokens per cache block


def main(argv: Optional[List[str]] = None) -> int:
    p = argparse.ArgumentParser(
        prog="trace_run", description="replay a trace of token ids")
    p.add_argument("--model", required=True,
                   help="folder with config.json and model.safetensors")
    p.add_argument("--dtype", choices=["bfloat16", "float32"],
                   default="bfloat16")
    p.add_argument("--out", required=True, help="folder for the logits")
    p.add_argument("--max-tokens", type=int, required=True,
                   help="most tokens that live requests hold at a time, each "
                        f"request rounded up to a multiple of {BLOCK}")
    p.add_argument("--device", default=None,
                   help="default: the GPU if there is one")
    args = p.parse_args(argv)

    import torch

    from fei_amd import ops
    from fei_amd.engine.config import get_spec
    from fei_amd.engine.step import StepEntry, StepRunner
    from fei_amd.models import model_class

    device = torch.device(args.device or
                          ("cuda:0" if torch.cuda.is_available() else "cpu"))
    if device.type == "cuda":
        ops.build_if_missing()
    spec = get_spec(args.model)
    cls = model_class(spec)
    if not getattr(cls, "step_cache", False):
        print(f"trace_run: {spec.arch} models do not run ragged steps",
              file=sys.stderr)
        return 2
    blocks = -(-args.max_tokens // BLOCK)
    longest = min(blocks * BLOCK, spec.max_positions or blocks * BLOCK)
    model = cls(spec, device, getattr(torch, args.dtype),
                max_seq_len=longest, weights=args.model)
    runner = StepRunner(model, num_blocks=blocks, num_slots=SLOTS,
                        block_size=BLOCK)

    live: Dict[str, int] = {}
    for line in sys.stdin:
        if not line.strip():
            continue
        req = json.loads(line)
        entries = []
        for e in req.get("entries", []):
            if not e["tokens"]:
                continue
            if e["id"] not in live:
                live[e["id"]] = runner.admit()
            entries.append(StepEntry(live[e["id"]], e["tokens"],
                                     e.get("want", [])))
        if entries:
            logits = runner.step(entries)
            if logits.shape[0]:
                data = logits.float().cpu().numpy().astype("<f4")
                with open(os.path.join(args.out, f"{req['step']}.f32"),
                          "wb") as f:
                    f.write(data.tobytes())
        for name in req.get("end", []):
            if name in live:
                runner.release(live.pop(name))
        print(f"done {req['step']}", flush=True)
    return 0


if __name__ == "__main__":
    raise SystemExit(main())
