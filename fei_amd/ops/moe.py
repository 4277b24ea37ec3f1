"""Mixtures of experts: sigmoid router, experts W_down relu(W_up h)^2.

Same dispatch rule as the rest of ``fei_amd.ops`` (kernels: csrc/moe.hip).
One or a few rows take one gemv per chosen expert; more rows are sorted by
expert on the device (``plan``) and go through grouped matrix products whose
tiles each belong to one expert.
"""

from __future__ import annotations

import ctypes
from typing import Tuple

import torch

from fei_amd.ops import reference as ref
from fei_amd.ops.mixers import (GainNormed, _f32, _gemv_rows, _lib, _p,
                                _stream, residual_linear)

_c = ctypes
_vp, _i, _f, _l = _c.c_void_p, _c.c_int, _c.c_float, _c.c_long

MAX_EXPERTS = 1024


def declare(lib: ctypes.CDLL) -> None:
    lib.fei_moe_route.argtypes = [_vp] * 3 + [_i] * 3 + [_f, _vp]
    lib.fei_moe_plan.argtypes = [_vp] * 5 + [_i] * 5 + [_vp]
    lib.fei_moe_gemm.argtypes = [_vp] * 6 + [_i] * 5 + [_vp]
    lib.fei_moe_add.argtypes = [_vp] * 4 + [_i] * 3 + [_f, _i, _vp]
    lib.fei_moe_up_gemv.argtypes = (
        [_vp] * 6 + [_i] + [_vp, _f] + [_i] * 5 + [_f, _vp])
    lib.fei_moe_out_gemv.argtypes = (
        [_vp, _vp, _l] + [_vp] * 5 + [_i] * 5 + [_f, _vp])


def check_moe_geometry(f) -> None:
    if f.experts > MAX_EXPERTS:
        raise ValueError(f"more than {MAX_EXPERTS} experts: {f}")


def route(logits: torch.Tensor, top: int, scale: float
          ) -> Tuple[torch.Tensor, torch.Tensor]:
    """Router logits [T, E] float32 -> chosen experts [T, top] int32 and their
    weights [T, top] float32."""
    if not logits.is_cuda:
        ids, w = ref.route(logits, top, scale)
        return ids.int(), w
    T, E = logits.shape
    ids = torch.empty(T, top, dtype=torch.int32, device=logits.device)
    w = torch.empty(T, top, dtype=torch.float32, device=logits.device)
    if T:
        _lib().fei_moe_route(_p(ids), _p(w), _p(logits), T, E, top, scale,
                             _stream())
    return ids, w


def residual_moe(x: torch.Tensor, h: GainNormed, router: torch.Tensor,
                 a: torch.Tensor, w_o: torch.Tensor, up: torch.Tensor,
                 down: torch.Tensor, f, mult: float) -> torch.Tensor:
    """x + mult * (a @ w_o^T + experts(h)), float32; x may be overwritten.
    ``router``: the rows' logits; up [E, ff, C], down [E, C, ff]."""
    T, C = x.shape
    E, ff, _ = up.shape
    if not x.is_cuda:
        ids, w = ref.route(router, f.top, f.scale)
        y = ref.moe(h.rows, ids, w, up, down)
        return residual_linear(x, a, w_o, mult) + mult * y
    if T == 0:
        return x
    dev, st, lib = x.device, _stream(), _lib()
    if _gemv_rows(T, C, up) and ff % 8 == 0 and a.shape[1] % 8 == 0:
        ids = torch.empty(T, f.top, dtype=torch.int32, device=dev)
        w = torch.empty(T, f.top, dtype=torch.float32, device=dev)
        act = torch.empty(T * f.top, ff, dtype=up.dtype, device=dev)
        fused = h.inside
        src = h.x if fused else h.rows
        lib.fei_moe_up_gemv(
            _p(act), _p(ids), _p(w), _p(router), _p(up), _p(src), int(fused),
            _p(h.norm.gain), h.norm.eps, T, E, f.top, ff, C, f.scale, st)
        own = T <= 2         # the output product of the mixer joins in
        if not own:
            x = residual_linear(x, a, w_o, mult)
        lib.fei_moe_out_gemv(
            _p(x), _p(a), a.stride(0), _p(w_o), _p(act), _p(ids), _p(w),
            _p(down), T, C, a.shape[1] if own else 0, ff, f.top, mult, st)
        return x
    ids, w = route(router, f.top, f.scale)
    n = T * f.top
    # rows of a tile of the grouped products
    big = up.dtype == torch.bfloat16 and C % 64 == 0 and ff % 64 == 0 \
        and n >= 32 * E
    rows = 128 if big else 32
    max_tiles = min(n, n // rows + E)
    meta = torch.empty(2 * n + 3 * max_tiles + 1, dtype=torch.int32,
                       device=dev)
    order, place = meta[:n], meta[n:2 * n]
    tiles, count = meta[2 * n:-1], meta[-1:]
    # order: row of every slot, slots sorted by expert; place: slot of (t, k)
    lib.fei_moe_plan(_p(order), _p(place), _p(tiles), _p(count), _p(ids),
                     n, E, f.top, rows, max_tiles, st)
    act = torch.empty(n, ff, dtype=up.dtype, device=dev)
    y = torch.empty(n, C, dtype=up.dtype, device=dev)
    bits = _f32(up) | (2 if big else 0)
    lib.fei_moe_gemm(_p(act), _p(h.rows), _p(up), _p(order), _p(tiles),
                     _p(count), max_tiles, ff, C, 1, bits, st)
    lib.fei_moe_gemm(_p(y), _p(act), _p(down), None, _p(tiles), _p(count),
                     max_tiles, C, ff, 0, bits, st)
    x = residual_linear(x, a, w_o, mult)
    lib.fei_moe_add(_p(x), _p(y), _p(place), _p(w), T, C, f.top, mult,
                    _f32(up), st)
    return x
