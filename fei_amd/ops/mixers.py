"""Ops of decoders made of unlike layers (models/tobarax.py, models/bokenex.py,
models/mixers.py).

Same dispatch rule as the rest of ``fei_amd.ops``: GPU tensors go to the HIP
kernels (csrc/hybrid.hip, latent_attn.hip, gla.hip), in bfloat16 or float32 by
the dtype of the rows; CPU tensors to the reference implementations.
"""

from __future__ import annotations

import ctypes
from typing import Optional, Tuple

import torch

from fei_amd.ops import reference as ref

_c = ctypes
_vp, _i, _f, _l = _c.c_void_p, _c.c_int, _c.c_float, _c.c_long

MAX_SPLITS = 64          # splits of a decode row's keys
TARGET_BLOCKS = 256      # workgroups of a decode attention launch


def declare(lib: ctypes.CDLL) -> None:
    lib.fei_norm_pair.argtypes = [_vp] * 5 + [_i, _i, _f, _i, _vp]
    lib.fei_cat_cast.argtypes = [_vp, _vp, _vp, _i, _i, _i, _vp]
    lib.fei_swiglu_rows.argtypes = [_vp, _l, _vp, _l, _i, _i, _i, _vp]
    lib.fei_softcap.argtypes = [_vp, _l, _f, _f, _vp]
    lib.fei_gemv_mix_in.argtypes = [_vp] * 5 + [_l] + [_i] * 4 + [_i, _vp]
    lib.fei_gemv_f32.argtypes = [_vp] * 4 + [_i] * 3 + [_i, _f, _f, _i, _vp]
    lib.fei_embed_pos.argtypes = [_vp] * 5 + [_i] * 3 + [_vp]
    lib.fei_relu2_rows.argtypes = [_vp, _l, _vp, _l, _i, _i, _i, _vp]
    lib.fei_gemv_gain.argtypes = [_vp] * 4 + [_f] + [_i] * 3 + [_vp]
    lib.fei_gemv_parallel_in.argtypes = (
        [_vp] * 5 + [_f] + [_vp, _l] + [_i] * 5 + [_vp])
    lib.fei_gemm_m8_parallel_in.argtypes = (
        [_vp] * 5 + [_l] + [_i] * 5 + [_vp])
    lib.fei_gemm_m8_f32.argtypes = [_vp] * 4 + [_i] * 4 + [_f, _f, _vp]
    lib.fei_latent_decode.argtypes = (
        [_vp, _l, _vp, _l] + [_vp] * 10 + [_i] * 8 +
        [_f, _i, _f, _i, _i, _i, _vp])
    lib.fei_latent_decode.restype = _i
    lib.fei_latent_append.argtypes = (
        [_vp, _l] + [_vp] * 6 + [_i] * 8 + [_f, _i, _vp])
    lib.fei_latent_gather.argtypes = [_vp] * 6 + [_i] * 7 + [_vp]
    lib.fei_window_prefill.argtypes = (
        [_vp, _l, _vp, _l] + [_vp] * 4 + [_i] * 6 + [_f, _i, _i, _vp])
    lib.fei_gla_decode.argtypes = (
        [_vp, _l, _vp, _vp, _vp, _l] + [_vp] * 5 + [_i] * 5 + [_f, _f, _i, _vp])
    lib.fei_gla_prefill.argtypes = (
        [_vp, _l, _vp, _l] + [_vp] * 5 + [_i, _vp, _i] + [_vp] * 4 +
        [_i] * 4 + [_f, _f, _i, _vp])


def _lib() -> ctypes.CDLL:
    from fei_amd import ops
    return ops.require_lib()


def _stream() -> int:
    from fei_amd import ops
    return ops._stream()


def _p(t: Optional[torch.Tensor]):
    return None if t is None else t.data_ptr()


def _f32(t: torch.Tensor) -> int:
    """Element switch of the kernels: 0 = bfloat16, 1 = float32."""
    if t.dtype == torch.float32:
        return 1
    if t.dtype != torch.bfloat16:
        raise TypeError(f"rows must be bfloat16 or float32, not {t.dtype}")
    return 0


# -- row-wise ops ----------------------------------------------------------------

def norm_pair(x: torch.Tensor, w1: torch.Tensor, w2: Optional[torch.Tensor],
              eps: float, dtype: torch.dtype
              ) -> Tuple[torch.Tensor, Optional[torch.Tensor]]:
    """x [T, C] float32 -> (norm(x) * w1, norm(x) * w2) in ``dtype``; the
    second is None without w2."""
    if not x.is_cuda:
        return ref.norm_pair(x, w1, w2, eps, dtype)
    x = x.contiguous()
    T, C = x.shape
    o1 = torch.empty(T, C, dtype=dtype, device=x.device)
    o2 = None if w2 is None else torch.empty_like(o1)
    if T:
        _lib().fei_norm_pair(_p(o1), _p(o2), _p(x), _p(w1), _p(w2), T, C, eps,
                             _f32(o1), _stream())
    return o1, o2


def cat_cast(x: torch.Tensor, y: torch.Tensor,
             dtype: torch.dtype) -> torch.Tensor:
    """[x; y] along columns, float32 -> ``dtype``."""
    if not x.is_cuda:
        return torch.cat([x, y], dim=-1).to(dtype)
    T, C = x.shape
    out = torch.empty(T, 2 * C, dtype=dtype, device=x.device)
    _lib().fei_cat_cast(_p(out), _p(x.contiguous()), _p(y.contiguous()), T, C,
                        _f32(out), _stream())
    return out


def embed_pos(tokens: torch.Tensor, pos: torch.Tensor, emb: torch.Tensor,
              pos_emb: torch.Tensor) -> torch.Tensor:
    """emb[tokens] + pos_emb[pos], float32 [T, C]."""
    if not emb.is_cuda:
        return emb[tokens.long()].float() + pos_emb[pos.long()].float()
    T, C = tokens.shape[0], emb.shape[1]
    out = torch.empty(T, C, dtype=torch.float32, device=emb.device)
    if tokens.dtype not in (torch.int32, torch.int64):
        raise TypeError(f"token ids are {tokens.dtype}")
    if T:
        _lib().fei_embed_pos(
            _p(out), _p(tokens.contiguous()), _p(pos), _p(emb), _p(pos_emb),
            T, C, _f32(emb) | (2 if tokens.dtype == torch.int64 else 0),
            _stream())
    return out


class GainNorm:
    """RMS norm with one gain for all columns."""

    def __init__(self, gain: torch.Tensor, width: int, eps: float):
        self.gain, self.eps = gain, eps
        # as a weight per column, for the norm of rows
        self.cols = gain.expand(width).contiguous()


class GainNormed:
    """Rows x (float32) under a GainNorm. The gain and the root mean square
    commute with a product, so a product of a row or two takes x as it is
    and makes the norm inside; the others take the normed ``rows``."""

    def __init__(self, x: torch.Tensor, norm: GainNorm, dtype: torch.dtype):
        self.x, self.norm, self.dtype = x, norm, dtype
        self._rows: Optional[torch.Tensor] = None

    @property
    def rows(self) -> torch.Tensor:
        if self._rows is None:
            self._rows, _ = norm_pair(self.x, self.norm.cols, None,
                                      self.norm.eps, self.dtype)
        return self._rows

    @property
    def inside(self) -> bool:
        """Whether products make the norm inside."""
        return (self.x.is_cuda and self.dtype == torch.bfloat16
                and self.x.shape[0] <= 2 and self.x.shape[1] % 8 == 0
                and self.x.shape[0] > 0)


def _gemv_rows(T: int, K: int, t: torch.Tensor) -> bool:
    return T in (1, 2, 4, 8) and K % 8 == 0 and t.dtype == torch.bfloat16


def _m8(T: int, K: int, t: torch.Tensor, *cols: int) -> bool:
    """Rows and sizes that the small matrix-core tile takes."""
    return (4 <= T <= 8 and K % 1024 == 0 and t.dtype == torch.bfloat16
            and all(n % 16 == 0 for n in cols))


def mix_in(n1: torch.Tensor, n2: Optional[torch.Tensor], w_in: torch.Tensor,
           n_mix: int, ff: int, act: torch.Tensor) -> torch.Tensor:
    """All products of a layer's input: returns n1 @ w_in[:n_mix]^T and writes
    silu(gate) * up of n2, gate and up being the next ``ff`` rows each, into
    ``act`` (a column range of a wider buffer)."""
    T, K = n1.shape
    if n1.is_cuda and _m8(T, K, n1, n_mix, 2 * ff):
        proj = torch.empty(T, n_mix, dtype=n1.dtype, device=n1.device)
        _lib().fei_gemm_m8(_p(proj), _p(n1), _p(w_in), T, n_mix, K, 0,
                           _stream())
        if ff:
            gu = torch.empty(T, 2 * ff, dtype=n1.dtype, device=n1.device)
            _lib().fei_gemm_m8(_p(gu), _p(n2), _p(w_in[n_mix:]), T, 2 * ff, K,
                               0, _stream())
            _lib().fei_swiglu_rows(_p(act), act.stride(0), _p(gu), 2 * ff, T,
                                   ff, 0, _stream())
        return proj
    if n1.is_cuda and _gemv_rows(T, K, n1):
        proj = torch.empty(T, n_mix, dtype=n1.dtype, device=n1.device)
        _lib().fei_gemv_mix_in(_p(proj), _p(act), _p(n1), _p(n2), _p(w_in),
                               act.stride(0), T, n_mix, ff, K, 1, _stream())
        return proj
    proj = torch.nn.functional.linear(n1, w_in[:n_mix])
    if ff:
        gu = torch.nn.functional.linear(n2, w_in[n_mix:])
        if n1.is_cuda:
            if T:
                _lib().fei_swiglu_rows(_p(act), act.stride(0), _p(gu),
                                       gu.stride(0), T, ff, _f32(gu),
                                       _stream())
        else:
            act.copy_(ref.swiglu(gu))
    return proj


def parallel_in(h: GainNormed, w_in: torch.Tensor, n_mix: int, ff: int,
                n_router: int, act: torch.Tensor
                ) -> Tuple[torch.Tensor, Optional[torch.Tensor]]:
    """All products of a parallel layer's input. The rows of ``w_in`` are
    n_mix of the mixer, whose products are returned, then either ``ff`` of a
    feed-forward, relu(.)^2 of which goes into ``act`` (a column range of a
    wider buffer), or ``n_router`` of a router, whose float32 logits are
    returned second (None without)."""
    x, norm = h.x, h.norm
    T, K = x.shape
    n = n_mix + ff + n_router
    gpu = x.is_cuda and h.dtype == torch.bfloat16
    if h.inside or (gpu and _m8(T, K, w_in, n)):
        proj = torch.empty(T, n_mix, dtype=h.dtype, device=x.device)
        router = torch.empty(T, n_router, dtype=torch.float32,
                             device=x.device) if n_router else None
        if h.inside:
            _lib().fei_gemv_parallel_in(
                _p(proj), _p(router), _p(x), _p(w_in), _p(norm.gain), norm.eps,
                _p(act), act.stride(0), T, n_mix, n_router, n, K, _stream())
        else:
            _lib().fei_gemm_m8_parallel_in(
                _p(proj), _p(router), _p(h.rows), _p(w_in), _p(act),
                act.stride(0), T, n_mix, n_router, n, K, _stream())
        return proj, router
    rows = h.rows
    proj = torch.nn.functional.linear(rows, w_in[:n_mix])
    if ff:
        up = torch.nn.functional.linear(rows, w_in[n_mix:])
        if not x.is_cuda:
            act.copy_(ref.square_relu(up))
        elif T:
            _lib().fei_relu2_rows(_p(act), act.stride(0), _p(up),
                                  up.stride(0), T, ff, _f32(up), _stream())
    router = _mm_f32(rows, w_in[n_mix:], None) if n_router else None
    return proj, router


def gain_logits(h: GainNormed, w: torch.Tensor) -> torch.Tensor:
    """normed rows @ w^T, float32."""
    if not h.inside:
        return logits_head(h.rows, w, 1.0, None)
    T, K = h.x.shape
    out = torch.empty(T, w.shape[0], dtype=torch.float32, device=w.device)
    _lib().fei_gemv_gain(_p(out), _p(h.x.contiguous()), _p(w),
                         _p(h.norm.gain), h.norm.eps, T, w.shape[0], K,
                         _stream())
    return out


def _mm_f32(a: torch.Tensor, w: torch.Tensor,
            add: Optional[torch.Tensor]) -> torch.Tensor:
    """a @ w^T (+ add) with a float32 result; a 2-d ``add`` may be
    overwritten with it."""
    if not a.is_cuda or a.dtype == torch.float32:
        y = torch.nn.functional.linear(a.float(), w.float())
        return y if add is None else add + y
    if add is None:
        return torch.mm(a, w.t(), out_dtype=torch.float32)
    if add.dim() == 1:
        return torch.addmm(add.expand(a.shape[0], -1), a, w.t(),
                           out_dtype=torch.float32)
    return torch.addmm(add, a, w.t(), out_dtype=torch.float32, out=add)


def residual_linear(x: torch.Tensor, a: torch.Tensor, w: torch.Tensor,
                    mult: float = 1.0) -> torch.Tensor:
    """x + mult * (a @ w^T), float32; x may be overwritten with it."""
    T, K = a.shape
    if a.is_cuda and _m8(T, K, a, w.shape[0]):
        _lib().fei_gemm_m8_f32(_p(x), _p(a), _p(w), None, T, w.shape[0], K, 1,
                               mult, 0.0, _stream())
        return x
    if a.is_cuda and _gemv_rows(T, K, a):
        _lib().fei_gemv_f32(_p(x), _p(a), _p(w), None, T, w.shape[0], K, 1,
                            mult, 0.0, 1, _stream())
        return x
    if not a.is_cuda or a.dtype == torch.float32:
        return x + mult * _mm_f32(a, w, None)
    return torch.addmm(x, a, w.t(), out_dtype=torch.float32, alpha=mult,
                       out=x)


def linear_f32(a: torch.Tensor, w: torch.Tensor,
               bias: torch.Tensor) -> torch.Tensor:
    """a @ w^T + bias, float32."""
    T, K = a.shape
    if a.is_cuda and _m8(T, K, a, w.shape[0]):
        out = torch.empty(T, w.shape[0], dtype=torch.float32, device=a.device)
        _lib().fei_gemm_m8_f32(_p(out), _p(a), _p(w), _p(bias), T, w.shape[0],
                               K, 0, 1.0, 0.0, _stream())
        return out
    if a.is_cuda and _gemv_rows(T, K, a):
        out = torch.empty(T, w.shape[0], dtype=torch.float32, device=a.device)
        _lib().fei_gemv_f32(_p(out), _p(a), _p(w), _p(bias), T, w.shape[0], K,
                            0, 1.0, 0.0, 1, _stream())
        return out
    return _mm_f32(a, w, bias)


def logits_head(y: torch.Tensor, w: torch.Tensor, scale: float,
                cap: Optional[float]) -> torch.Tensor:
    """(y @ w^T) * scale, then cap * tanh(. / cap); float32."""
    T, K = y.shape
    if not y.is_cuda:
        return ref.softcap_logits(_mm_f32(y, w, None), scale, cap)
    c = float(cap or 0.0)
    if _m8(T, K, y, w.shape[0]):
        out = torch.empty(T, w.shape[0], dtype=torch.float32, device=y.device)
        _lib().fei_gemm_m8_f32(_p(out), _p(y), _p(w), None, T, w.shape[0], K,
                               0, scale, c, _stream())
        return out
    if _gemv_rows(T, K, y):
        out = torch.empty(T, w.shape[0], dtype=torch.float32, device=y.device)
        _lib().fei_gemv_f32(_p(out), _p(y), _p(w), None, T, w.shape[0], K, 0,
                            scale, c, 1, _stream())
        return out
    out = _mm_f32(y, w, None)
    if T:
        _lib().fei_softcap(_p(out), out.numel(), scale, c, _stream())
    return out


# -- latent attention --------------------------------------------------------------

def check_latent_geometry(m) -> None:
    """Largest sizes the kernels are built for."""
    if m.dim + m.rot_dim > 256 or m.vdim > 256 or m.kv_rank > 1024 \
            or m.row_width > 1088:
        raise ValueError(f"latent attention sizes out of range: {m}")


def _dst(batch, lo: int, hi: Optional[int], block_size: int) -> torch.Tensor:
    """Physical cache row of batch rows lo .. hi-1."""
    pos = batch.pos[lo:hi].long()
    blk = batch.table[batch.row_seq[lo:hi].long(), pos // block_size]
    return blk.long() * block_size + pos % block_size


def _keys(batch, seq: int, lo: int, hi: int, rows, block_size: int):
    """Cached rows of positions lo .. hi-1 of a sequence."""
    p = torch.arange(lo, hi)
    blk = batch.table[seq].long()[p // block_size]
    return rows[blk * block_size + p % block_size]


def _latent_out(o, proj, m, out) -> None:
    g = proj[:, m.in_rows - m.heads * m.vdim:].float()
    out.copy_((o.flatten(1) * torch.sigmoid(g)).to(out.dtype))


def latent_attn_decode(proj, out, m, w, rot, batch, rows,
                       block_size: int) -> None:
    """One new token per sequence: cache its row, attend, gate. proj
    [B, m.in_rows] (q | latent and rotated key | gate), out [B, H*vdim]."""
    if not proj.is_cuda:
        n = batch.n_dec
        q = ref.latent_append(proj, m, w.norm, rot, w.eps, batch.pos[:n],
                              _dst(batch, 0, n, block_size), rows)
        o = torch.empty(n, m.heads, m.vdim)
        for b in range(n):
            p = int(batch.pos[b])
            k0 = 0 if m.window is None else max(0, p - m.window + 1)
            o[b] = ref.latent_attend(
                q[b:b + 1], batch.pos[b:b + 1],
                _keys(batch, b, k0, p + 1, rows, block_size), k0, m, w.uk,
                w.uv, m.scale)[0]
        _latent_out(o, proj, m, out)
        return
    B, dev = proj.shape[0], proj.device
    W = batch.table.shape[1]
    n_max = W * block_size
    if m.window is not None:
        n_max = min(n_max, m.window)
    groups = B * -(-m.heads // 32)
    splits = max(1, min(MAX_SPLITS, -(-n_max // 32),
                        -(-TARGET_BLOCKS // groups)))
    per_split = -(-n_max // splits)
    tile = 32 if per_split <= 48 else 64
    qa = torch.empty(B, m.heads, m.row_width, dtype=proj.dtype, device=dev)
    part_o = torch.empty(B, m.heads, splits, m.kv_rank, dtype=torch.float32,
                         device=dev)
    part_ml = torch.empty(B, m.heads, splits, 2, dtype=torch.float32,
                          device=dev)
    rc = _lib().fei_latent_decode(
        _p(out), out.stride(0), _p(proj), proj.stride(0), _p(w.uk), _p(w.uv),
        _p(w.norm), _p(rot), _p(rows), _p(batch.pos), _p(batch.table), _p(qa),
        _p(part_o), _p(part_ml), B, W, block_size.bit_length() - 1, m.heads,
        m.dim, m.rot_dim, m.vdim, m.kv_rank, m.scale, m.window or 0, w.eps,
        splits, tile, _f32(proj), _stream())
    if rc:
        raise ValueError(f"no decode tile for {m}")


def latent_attn_prefill(proj, out, m, w, rot, batch, rows,
                        block_size: int) -> None:
    """Prompt portions: rows n_dec .. of proj and out."""
    n = batch.n_dec
    if not proj.is_cuda:
        p_, o_ = proj[n:], out[n:]
        q = ref.latent_append(p_, m, w.norm, rot, w.eps, batch.pos[n:],
                              _dst(batch, n, None, block_size), rows)
        o = torch.empty(p_.shape[0], m.heads, m.vdim)
        for i, (row, cnt, pos0) in enumerate(batch.portions):
            k0 = 0 if m.window is None else max(0, pos0 - m.window + 1)
            at = slice(row - n, row - n + cnt)
            o[at] = ref.latent_attend(
                q[at], batch.pos[row:row + cnt],
                _keys(batch, n + i, k0, pos0 + cnt, rows, block_size), k0, m,
                w.uk, w.uv, m.scale)
        _latent_out(o, p_, m, o_)
        return
    lib, dev, st = _lib(), proj.device, _stream()
    W, bs_log = batch.table.shape[1], block_size.bit_length() - 1
    f32, T = _f32(proj), proj.shape[0] - n
    pr = proj[n:]
    lib.fei_latent_append(
        _p(pr), proj.stride(0), _p(rows), _p(w.norm), _p(rot),
        _p(batch.pos[n:]), _p(batch.row_seq[n:]), _p(batch.table), T, W,
        bs_log, m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, w.eps, f32, st)
    spans, n_keys, tiles, owner = batch.key_plan(m.window)
    c = torch.empty(n_keys, m.kv_rank, dtype=proj.dtype, device=dev)
    kr = torch.empty(n_keys, m.rot_dim, dtype=proj.dtype, device=dev)
    lib.fei_latent_gather(_p(c), _p(kr), _p(rows), _p(owner), _p(spans),
                          _p(batch.table), n_keys, W, bs_log, n, m.kv_rank,
                          m.rot_dim, f32, st)
    kv = torch.nn.functional.linear(c, w.ukv)
    lib.fei_window_prefill(
        _p(out), out.stride(0), _p(proj), proj.stride(0), _p(kv), _p(kr),
        _p(spans), _p(tiles), tiles.shape[0], m.heads, m.dim, m.rot_dim,
        m.vdim, m.kv_rank, m.scale, m.window or 0, f32, st)


# -- gated linear attention ----------------------------------------------------------

def check_gla_geometry(m) -> None:
    if m.dim > 256 or m.vdim > 512 or m.gate_rank > 128:
        raise ValueError(f"gated linear attention sizes out of range: {m}")


def _gla_split(proj, m, w):
    """q (scaled), k, v as [T, H, .] float32, gate columns, log decay."""
    T, a, b = proj.shape[0], m.heads * m.dim, m.heads * m.vdim
    q, k, v, g, a1 = proj.split([a, a, b, b, m.gate_rank], dim=-1)
    ld = ref.gla_log_decay(a1, w.a2, w.bias, m.tau)
    return (q.float().view(T, m.heads, m.dim) * m.dim ** -0.5,
            k.float().view(T, m.heads, m.dim),
            v.float().view(T, m.heads, m.vdim), g,
            ld.view(T, m.heads, m.dim))


def _gla_cpu(proj, out, m, w, state, fresh: bool) -> None:
    q, k, v, g, ld = _gla_split(proj, m, w)
    o, S = ref.gla_scan(q, k, v, ld, torch.zeros_like(state) if fresh
                        else state)
    state.copy_(S)
    out.copy_(ref.gla_gate_out(o, g, w.norm, w.eps).to(out.dtype))


def gla_decode(proj, out, m, w, batch, states) -> None:
    """One new token per sequence. proj [B, m.in_rows] (q | k | v | gate |
    low-rank decay input), out [B, H*vdim], states [slots+1, H, vdim, dim]."""
    if not proj.is_cuda:
        for b in range(batch.n_dec):
            _gla_cpu(proj[b:b + 1], out[b:b + 1], m, w,
                     states[int(batch.slots[b])], int(batch.pos[b]) == 0)
        return
    B = proj.shape[0]
    o = torch.empty(B, m.heads * m.vdim, dtype=torch.float32,
                    device=proj.device)
    _lib().fei_gla_decode(
        _p(out), out.stride(0), _p(o), _p(states), _p(proj), proj.stride(0),
        _p(w.a2), _p(w.bias), _p(w.norm), _p(batch.pos), _p(batch.slots), B,
        m.heads, m.dim, m.vdim, m.gate_rank, m.tau, w.eps, _f32(proj),
        _stream())


def gla_prefill(proj, out, m, w, batch, states) -> None:
    """Prompt portions: rows n_dec .. of proj and out."""
    if not proj.is_cuda:
        for i, (row, n, pos0) in enumerate(batch.portions):
            _gla_cpu(proj[row:row + n], out[row:row + n], m, w,
                     states[int(batch.slots[batch.n_dec + i])], pos0 == 0)
        return
    dev = proj.device
    chunks, spans = batch.chunk_plan()
    n = chunks.shape[0]
    f = dict(dtype=torch.float32, device=dev)
    G = torch.empty(proj.shape[0], m.heads * m.dim, **f)
    U = torch.empty(n, m.heads, m.vdim, m.dim, **f)
    A = torch.empty(n, m.heads, 64, 64, **f)
    _lib().fei_gla_prefill(
        _p(out), out.stride(0), _p(proj), proj.stride(0), _p(w.a2),
        _p(w.bias), _p(w.norm), _p(states), _p(chunks), n, _p(spans),
        spans.shape[0], _p(batch.slots), _p(G), _p(U), _p(A), m.heads, m.dim,
        m.vdim, m.gate_rank, m.tau, w.eps, _f32(proj), _stream())
