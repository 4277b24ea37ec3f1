"""Grouped-query attention with sigmoid key weights (models/mixers.py).

Same dispatch rule as the rest of ``fei_amd.ops``: GPU tensors go to the HIP
kernels (csrc/sigmoid_attn.hip), CPU tensors to the reference operations.
A cached row is [keys (kv_heads * dim) | values (kv_heads * vdim)]; a state
holds the last ``conv`` projected rows, that of position p at p % conv.
"""

from __future__ import annotations

import ctypes

import torch

from fei_amd.ops import reference as ref
from fei_amd.ops.mixers import _dst, _f32, _keys, _lib, _p, _stream

_c = ctypes
_vp, _i, _f, _l = _c.c_void_p, _c.c_int, _c.c_float, _c.c_long

SPLIT_KEYS = 128         # least keys of a decode split: 32 for each wave
MAX_SPLITS = 64
TARGET_BLOCKS = 512      # workgroups of a decode launch


def declare(lib: ctypes.CDLL) -> None:
    lib.fei_sig_decode.argtypes = (
        [_vp, _l, _vp, _vp, _l] + [_vp] * 9 + [_i] * 9 + [_f, _i, _f, _i, _i,
                                                          _vp])
    lib.fei_sig_conv.argtypes = (
        [_vp, _vp, _l] + [_vp] * 10 + [_i] * 10 + [_f, _i, _vp])
    lib.fei_sig_prefill.argtypes = (
        [_vp, _l] + [_vp] * 6 + [_i] * 9 + [_f, _i, _vp])


def check_sigmoid_geometry(m) -> None:
    """Largest sizes the kernels are built for."""
    if m.dim > 256 or m.vdim > 256:
        raise ValueError(f"attention sizes out of range: {m}")


def _conv_norm_cpu(u, m, w, state, pos0: int):
    """Convolution and norms of a sequence's next projections u [n, rows];
    keeps the last ``conv`` of them. Returns q [n, H, dim] and cache rows."""
    n, taps = u.shape[0], m.conv
    u = u.float()
    first = torch.zeros(taps - 1, u.shape[1])
    for a in range(1, taps):
        if pos0 - a >= 0:
            first[taps - 1 - a] = state[(pos0 - a) % taps]
    if state is not None:
        for i in range(max(0, n - taps), n):
            state[(pos0 + i) % taps] = u[i]
    y = ref.short_conv(u, first, w.conv)
    q, k, v = y.split([m.heads * m.dim, m.kv_heads * m.dim,
                       m.kv_heads * m.vdim], dim=-1)
    q = ref.rms(q.view(n, m.heads, m.dim), w.eps) * w.qn
    k = ref.rms(k.view(n, m.kv_heads, m.dim), w.eps) * w.kn
    return q, torch.cat([k.flatten(1), v], dim=-1)


def _portion_cpu(proj, out, m, w, batch, rows, states, block_size, seq: int,
                 row: int, pos0: int) -> None:
    n = proj.shape[0]
    state = None if states is None else states[int(batch.slots[seq])]
    q, kv = _conv_norm_cpu(proj, m, w, state, pos0)
    rows[_dst(batch, row, row + n, block_size)] = kv.to(rows.dtype)
    k0 = 0 if m.window is None else max(0, pos0 - m.window + 1)
    o = ref.sigmoid_attend(q.to(rows.dtype).float(),
                           batch.pos[row:row + n],
                           _keys(batch, seq, k0, pos0 + n, rows, block_size),
                           k0, m, w.bias)
    out.copy_(o.flatten(1).to(out.dtype))


def sigmoid_attn_decode(proj, out, m, w, batch, rows, states,
                        block_size: int) -> None:
    """One new token per sequence: convolution, norms, cache row, state,
    attention. proj [B, m.in_rows] (q | k | v), out [B, H*vdim]."""
    B = proj.shape[0]
    if not proj.is_cuda:
        for b in range(B):
            _portion_cpu(proj[b:b + 1], out[b:b + 1], m, w, batch, rows,
                         states, block_size, b, b, int(batch.pos[b]))
        return
    dev, W = proj.device, batch.table.shape[1]
    n_max = W * block_size
    if m.window is not None:
        n_max = min(n_max, m.window)
    # a split starts at a multiple of 32 keys, so a window may touch 31 more
    per_head = B * m.kv_heads * -(-(m.heads // m.kv_heads) // 16)
    splits = max(1, min(MAX_SPLITS, -(-(n_max + 31) // SPLIT_KEYS),
                        -(-TARGET_BLOCKS // per_head)))
    part = torch.empty(B, splits, m.heads * m.vdim, dtype=torch.float32,
                       device=dev)
    _lib().fei_sig_decode(
        _p(out), out.stride(0), _p(part), _p(proj), proj.stride(0), _p(rows),
        _p(states), _p(w.conv), _p(w.qn), _p(w.kn), _p(w.bias),
        _p(batch.pos), _p(batch.slots), _p(batch.table), B, W,
        block_size.bit_length() - 1, m.heads, m.kv_heads, m.dim, m.vdim,
        m.conv, m.window or 0, m.scale, splits, w.eps, SPLIT_KEYS,
        _f32(proj), _stream())


def sigmoid_attn_prefill(proj, out, m, w, batch, rows, states,
                         block_size: int) -> None:
    """Prompt portions: rows n_dec .. of proj and out."""
    n = batch.n_dec
    if not proj.is_cuda:
        for i, (row, cnt, pos0) in enumerate(batch.portions):
            at = slice(row, row + cnt)
            _portion_cpu(proj[at], out[at], m, w, batch, rows, states,
                         block_size, n + i, row, pos0)
        return
    spans, tiles = batch.span_plan()
    T, W = proj.shape[0] - n, batch.table.shape[1]
    bs_log, st = block_size.bit_length() - 1, _stream()
    q = torch.empty(T, m.heads * m.dim, dtype=proj.dtype, device=proj.device)
    _lib().fei_sig_conv(
        _p(q), _p(proj), proj.stride(0), _p(rows), _p(states), _p(w.conv),
        _p(w.qn), _p(w.kn), _p(spans), _p(batch.row_seq), _p(batch.pos),
        _p(batch.slots), _p(batch.table), T, n, spans.shape[0], W, bs_log,
        m.heads, m.kv_heads, m.dim, m.vdim, m.conv, w.eps, _f32(proj), st)
    _lib().fei_sig_prefill(
        _p(out), out.stride(0), _p(q), _p(rows), _p(w.bias), _p(spans),
        _p(tiles), _p(batch.table), tiles.shape[0], n, W, bs_log, m.heads,
        m.kv_heads, m.dim, m.vdim, m.window or 0, m.scale, _f32(proj), st)
