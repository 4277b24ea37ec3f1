"""Prefill and decode throughput of several models side by side.

`python bench.py --compare tobarax-1b,llama3-1b` runs every model at the same
prompt lengths and batches, with random weights, and prints one JSON line per
model and batch.
"""

from __future__ import annotations

import json
import statistics
import time
from typing import Dict, List, Sequence

import torch

from fei_amd.engine.config import get_spec
from fei_amd.engine.engine import LocalEngine


def _sync(engine: LocalEngine) -> None:
    if engine.is_gpu:
        torch.cuda.synchronize(engine.device)


def measure(model: str, batch: int, prompts: Sequence[int], steps: int,
            repeats: int = 5) -> Dict[str, object]:
    """Median times over ``repeats``; a prefill includes the first token's
    sampling, a decode step the whole captured step."""
    spec = get_spec(model)
    max_seq = min(spec.max_seq_len, max(prompts) + (repeats + 1) * steps + 16)
    engine = LocalEngine.create(model, batch_size=batch, max_seq_len=max_seq)
    rng = torch.Generator().manual_seed(7)
    out: Dict[str, object] = {"model": model, "batch": batch,
                              "dtype": str(engine.dtype).split(".")[-1],
                              "params_gb": round(
                                  engine.model.param_bytes() / 1e9, 3)}
    for n in prompts:
        ids: List[int] = torch.randint(4, 260, (n,), generator=rng).tolist()
        times = []
        for _ in range(repeats + 1):
            _sync(engine)
            t = time.perf_counter()
            engine.prefill(ids)
            _sync(engine)
            times.append(time.perf_counter() - t)
        ms = statistics.median(times[1:]) * 1e3
        out[f"prefill_{n}_ms"] = round(ms, 3)
        out[f"prefill_{n}_tok_s"] = round(batch * n / ms * 1e3)
        times = []
        for _ in range(repeats + 1):
            _sync(engine)
            t = time.perf_counter()
            for _ in range(steps):
                if engine._graph is not None:
                    engine._graph.replay()
                else:
                    engine._decode_step()
            _sync(engine)
            times.append((time.perf_counter() - t) / steps)
        ms = statistics.median(times[1:]) * 1e3
        out[f"decode_{n}_ms"] = round(ms, 4)
        out[f"decode_{n}_tok_s"] = round(batch / ms * 1e3, 1)
    engine.shutdown()
    return out


def compare(models: Sequence[str], batches: Sequence[int],
            prompts: Sequence[int], steps: int) -> None:
    for batch in batches:
        for model in models:
            print(json.dumps(measure(model, batch, prompts, steps)),
                  flush=True)
