"""Token mixers of decoders made of unlike layers.

A mixer is given the stacked projections of its input (``IN`` names them in
row order), writes its output rows, and keeps what later tokens need in its
layer run's part of a HybridCache. Sizes and constants come from its spec.
"""

from __future__ import annotations

from typing import Callable, Dict, Optional, Tuple

import torch

from fei_amd import ops
from fei_amd.engine.config import (GLASpec, LatentAttentionSpec,
                                   SigmoidAttentionSpec)

Get = Callable[[str], torch.Tensor]


class Mixer:
    IN: Tuple[str, ...] = ()
    row_width: Optional[int] = None       # cached values per token
    state_shape: Optional[Tuple[int, ...]] = None   # state per sequence

    @staticmethod
    def shapes(m, width: int) -> Dict[str, tuple]:
        """Shapes of the mixer's tensors, output product included."""
        raise NotImplementedError

    def own_weights(self) -> Dict[str, torch.Tensor]:
        """The tensors that are neither in the stacked input product nor in
        the output product."""
        raise NotImplementedError

    def run(self, proj: torch.Tensor, out: torch.Tensor, batch, cache,
            run: int, rot: Dict) -> None:
        raise NotImplementedError


class LatentAttention(Mixer):
    """Attention over cached latents, with a rotated key part shared by the
    heads, a sliding window, and a sigmoid gate on the output."""

    IN = ("q", "dkv", "g")

    @staticmethod
    def shapes(m: LatentAttentionSpec, width: int) -> Dict[str, tuple]:
        return {"q": (m.heads * (m.dim + m.rot_dim), width),
                "dkv": (m.row_width, width),
                "g": (m.heads * m.vdim, width),
                "dkv.norm": (m.kv_rank,),
                "uk": (m.heads * m.dim, m.kv_rank),
                "uv": (m.heads * m.vdim, m.kv_rank),
                "o": (width, m.heads * m.vdim)}

    def __init__(self, m: LatentAttentionSpec, eps: float, mat: Get, vec: Get):
        ops.check_latent_geometry(m)
        self.m, self.eps = m, eps
        self.norm = vec("dkv.norm")
        self.ukv = torch.cat([mat("uk"), mat("uv")], dim=0).contiguous()
        self.uk = self.ukv[:m.heads * m.dim]
        self.uv = self.ukv[m.heads * m.dim:]
        self.row_width = m.row_width

    def own_weights(self) -> Dict[str, torch.Tensor]:
        return {"dkv.norm": self.norm, "uk": self.uk, "uv": self.uv}

    def run(self, proj, out, batch, cache, run, rot) -> None:
        m = self.m
        args = (m, self, rot[m.rot_dim, m.rot_base], batch, cache.rows[run],
                cache.block_size)
        n = batch.n_dec
        if n:
            ops.latent_attn_decode(proj[:n], out[:n], *args)
        if batch.portions:
            ops.latent_attn_prefill(proj, out, *args)


class GatedLinearAttention(Mixer):
    """Linear attention with a per-key-channel decay from a low-rank gate, a
    per-head norm and a silu gate on the output."""

    IN = ("q", "k", "v", "g", "a1")

    @staticmethod
    def shapes(m: GLASpec, width: int) -> Dict[str, tuple]:
        return {"q": (m.heads * m.dim, width), "k": (m.heads * m.dim, width),
                "v": (m.heads * m.vdim, width),
                "g": (m.heads * m.vdim, width),
                "a1": (m.gate_rank, width),
                "a2": (m.heads * m.dim, m.gate_rank),
                "a2.b": (m.heads * m.dim,), "norm": (m.vdim,),
                "o": (width, m.heads * m.vdim)}

    def __init__(self, m: GLASpec, eps: float, mat: Get, vec: Get):
        ops.check_gla_geometry(m)
        self.m, self.eps = m, eps
        self.norm, self.bias = vec("norm"), vec("a2.b")
        self.a2 = vec("a2")             # small, and feeds the recurrence
        # value-major, so that a value channel's keys are contiguous
        self.state_shape = (m.heads, m.vdim, m.dim)

    def own_weights(self) -> Dict[str, torch.Tensor]:
        return {"norm": self.norm, "a2.b": self.bias, "a2": self.a2}

    def run(self, proj, out, batch, cache, run, rot) -> None:
        args = (self.m, self, batch, cache.states[run])
        n = batch.n_dec
        if n:
            ops.gla_decode(proj[:n], out[:n], *args)
        if batch.portions:
            ops.gla_prefill(proj, out, *args)


class SigmoidAttention(Mixer):
    """Grouped-query attention with sigmoid key weights, a logarithmic
    distance bias and a sliding window, behind a short convolution over time
    and query/key norms. A cached row is the normed keys and the values; the
    state is the last ``conv`` projections, that of position p at p % conv."""

    IN = ("q", "k", "v")

    @staticmethod
    def shapes(m: SigmoidAttentionSpec, width: int) -> Dict[str, tuple]:
        nq, nk, nv = m.heads * m.dim, m.kv_heads * m.dim, m.kv_heads * m.vdim
        return {"q": (nq, width), "k": (nk, width), "v": (nv, width),
                "q.conv": (nq, m.conv), "k.conv": (nk, m.conv),
                "v.conv": (nv, m.conv), "q.norm": (m.dim,),
                "k.norm": (m.dim,), "r1": (m.heads,), "r2": (m.heads,),
                "pb": (m.heads,), "o": (width, m.heads * m.vdim)}

    def __init__(self, m: SigmoidAttentionSpec, eps: float, mat: Get,
                 vec: Get):
        ops.check_sigmoid_geometry(m)
        self.m, self.eps = m, eps
        self.qn, self.kn = vec("q.norm"), vec("k.norm")
        # per head: r1, r2, pb
        self.bias = torch.stack([vec("r1"), vec("r2"), vec("pb")]).contiguous()
        # tap-major, so that the channels of a tap are contiguous
        self.conv = torch.cat([vec(n + ".conv") for n in self.IN]).t() \
            .contiguous()
        self.row_width = m.row_width
        if m.conv > 1:
            self.state_shape = (m.conv, m.in_rows)

    def own_weights(self) -> Dict[str, torch.Tensor]:
        m = self.m
        cq, ck, cv = self.conv.t().split(
            [m.heads * m.dim, m.kv_heads * m.dim, m.kv_heads * m.vdim])
        return {"q.norm": self.qn, "k.norm": self.kn, "r1": self.bias[0],
                "r2": self.bias[1], "pb": self.bias[2], "q.conv": cq,
                "k.conv": ck, "v.conv": cv}

    def run(self, proj, out, batch, cache, run, rot) -> None:
        args = (self.m, self, batch, cache.rows[run], cache.states[run],
                cache.block_size)
        n = batch.n_dec
        if n:
            ops.sigmoid_attn_decode(proj[:n], out[:n], *args)
        if batch.portions:
            ops.sigmoid_attn_prefill(proj, out, *args)


MIXERS = {"latent_attention": LatentAttention, "gla": GatedLinearAttention,
          "attention": SigmoidAttention}
