"""What decoders that run RaggedBatches over a HybridCache have in common:
weights in a model folder, the cache, sizes.

A subclass gives ``_shapes`` (tensors by their name in a folder), ``_random``,
``_set_weights``, ``state_dict_full``, ``mixers`` (one per layer run, in
execution order) and ``forward``, which runs one RaggedBatch
(engine/step.py): prompts, portions of them and decoding sequences, in any
mixture. With single tokens only, nothing in a forward may depend on host
values, so that the step can be captured into a hipGraph.
"""

from __future__ import annotations

import json
import os
from typing import Callable, Dict, List, Optional

import torch

from fei_amd.engine.kv_cache import HybridCache
from fei_amd.models.mixers import Mixer
from fei_amd.parallel.pg import ParallelContext

Get = Callable[[str], torch.Tensor]


class StepModel:
    step_cache = True                   # runs RaggedBatches over a HybridCache

    def __init__(self, spec, device: torch.device,
                 dtype: torch.dtype = torch.bfloat16,
                 tp: Optional[ParallelContext] = None, seed: int = 1234,
                 max_seq_len: Optional[int] = None,
                 weights: Optional[str] = None):
        if tp is not None and tp.is_distributed:
            raise ValueError(f"{spec.name}: tensor parallelism is not "
                             "available for this architecture")
        self.spec = spec
        self.device = torch.device(device)
        self.dtype = dtype
        self.tp = tp or ParallelContext()
        self.tp_size = 1
        self._set_weights(self._read(weights) if weights
                          else self._random(seed))
        # a state holds exactly the tokens it has read: it cannot go back
        self.recurrent = any(m.state_shape is not None for m in self.mixers())
        self.resize(max_seq_len or spec.max_seq_len)

    def resize(self, max_seq_len: int) -> None:
        """Positions up to ``max_seq_len`` - 1 can be run from now on."""
        most = self.spec.max_positions
        if most is not None and max_seq_len > most:
            raise ValueError(f"{self.spec.name} has {most} positions, "
                             f"{max_seq_len} asked for")
        self.max_seq_len = max_seq_len

    # -- the subclass's ----------------------------------------------------------

    def mixers(self) -> List[Mixer]:
        raise NotImplementedError

    def _shapes(self) -> Dict[str, tuple]:
        raise NotImplementedError

    def _random(self, seed: int) -> Get:
        raise NotImplementedError

    def _set_weights(self, get: Get) -> None:
        raise NotImplementedError

    def state_dict_full(self) -> Dict[str, torch.Tensor]:
        """Tensors under their names in a model folder."""
        raise NotImplementedError

    def forward(self, batch, cache: HybridCache, on_run=None) -> torch.Tensor:
        raise NotImplementedError

    # -- weights -------------------------------------------------------------

    def _read(self, path: str) -> Get:
        """Tensors of a model folder, one at a time; names and shapes have to
        be exactly those of the spec."""
        from safetensors import safe_open

        f = safe_open(os.path.join(path, "model.safetensors"), framework="pt")
        shapes = self._shapes()
        names = set(f.keys())
        if names != set(shapes):
            raise ValueError(
                f"{path}: missing tensors {sorted(set(shapes) - names)[:4]}, "
                f"unknown tensors {sorted(names - set(shapes))[:4]}")

        def get(name: str) -> torch.Tensor:
            t = f.get_tensor(name)
            if tuple(t.shape) != tuple(shapes[name]):
                raise ValueError(f"{path}: {name} has shape {tuple(t.shape)},"
                                 f" expected {tuple(shapes[name])}")
            return t.to(self.device)
        return get

    def load_weights(self, path: str) -> None:
        self._set_weights(self._read(path))

    def save_weights(self, path: str) -> None:
        """Write a model folder (bfloat16, as such folders are)."""
        from safetensors.torch import save_file

        os.makedirs(path, exist_ok=True)
        save_file({k: v.to(torch.bfloat16).contiguous().cpu()
                   for k, v in self.state_dict_full().items()},
                  os.path.join(path, "model.safetensors"))
        with open(os.path.join(path, "config.json"), "w",
                  encoding="utf-8") as f:
            json.dump(self.spec.to_config(), f, indent=1)

    def param_bytes(self) -> int:
        return sum(t.numel() * t.element_size()
                   for t in self.state_dict_full().values())

    # -- cache -----------------------------------------------------------------

    def new_cache(self, num_blocks: int, num_slots: int,
                  block_size: int = 64) -> HybridCache:
        mixers = self.mixers()
        return HybridCache(
            [m.row_width for m in mixers], [m.state_shape for m in mixers],
            num_blocks, num_slots, block_size, self.device, self.dtype)

    def cache_bytes_per_token(self) -> int:
        el = torch.empty(0, dtype=self.dtype).element_size()
        return el * sum(m.row_width or 0 for m in self.mixers())
