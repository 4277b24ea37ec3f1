"""Feed-forwards of decoders made of unlike layers.

``IN`` names the tensors whose rows join the layer's stacked input product,
``OUT`` those whose columns join its stacked output product; the rest are the
feed-forward's own (a mixture of experts keeps its experts stacked).
"""

from __future__ import annotations

from typing import Callable, Dict, Tuple

import torch

from fei_amd import ops
from fei_amd.engine.config import DenseSpec, MoESpec

Get = Callable[[str], torch.Tensor]


class FeedForward:
    IN: Tuple[str, ...] = ()
    OUT: Tuple[str, ...] = ()
    act_cols = 0         # activations in the stacked output product
    router_rows = 0      # float32 rows of the stacked input product

    @staticmethod
    def shapes(f, width: int) -> Dict[str, tuple]:
        raise NotImplementedError

    def own_weights(self) -> Dict[str, torch.Tensor]:
        return {}


class SquaredReluFF(FeedForward):
    """W_down relu(W_up h)^2, wholly inside the layer's stacked products."""

    IN, OUT = ("up",), ("down",)

    def __init__(self, f: DenseSpec, mat: Get):
        self.f = f
        self.act_cols = f.ff

    @staticmethod
    def shapes(f: DenseSpec, width: int) -> Dict[str, tuple]:
        return {"up": (f.ff, width), "down": (width, f.ff)}


class MixtureOfExperts(FeedForward):
    """Experts of the same form, a few of them per token by sigmoid scores."""

    IN = ("router",)

    def __init__(self, f: MoESpec, mat: Get):
        ops.check_moe_geometry(f)
        self.f = f
        self.router_rows = f.experts
        self.up, self.down = (
            torch.stack([mat(f"e{e}.{n}") for e in range(f.experts)])
            for n in ("up", "down"))

    @staticmethod
    def shapes(f: MoESpec, width: int) -> Dict[str, tuple]:
        out: Dict[str, tuple] = {"router": (f.experts, width)}
        for e in range(f.experts):
            out[f"e{e}.up"] = (f.ff, width)
            out[f"e{e}.down"] = (width, f.ff)
        return out

    def own_weights(self) -> Dict[str, torch.Tensor]:
        return {f"e{e}.{n}": t[e] for n, t in (("up", self.up),
                                               ("down", self.down))
                for e in range(self.f.experts)}


FEED_FORWARDS = {"dense": SquaredReluFF, "moe": MixtureOfExperts}
