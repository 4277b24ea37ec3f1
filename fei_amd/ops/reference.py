"""Pure-PyTorch reference implementations of every engine op.

These define the *semantics* each HIP kernel must reproduce:
  - used directly on CPU (tests, tiny models, gloo multi-process tests)
  - GPU numerics tests compare the HIP kernels against these in fp32
    (tests/test_ops_gpu.py)

Shapes use B=batch, S=sequence, H/Hq/Hkv=heads, D=head_dim, C=hidden.
KV caches are contiguous ``[B, Hkv, max_seq, D]``.
"""

from __future__ import annotations

import math
from typing import Optional, Tuple

import torch


# -- normalisation -----------------------------------------------------------

def rmsnorm(x: torch.Tensor, weight: torch.Tensor, eps: float = 1e-5) -> torch.Tensor:
    """RMSNorm over the last dim; accumulate in fp32, output in x.dtype."""
    xf = x.float()
    var = xf.pow(2).mean(dim=-1, keepdim=True)
    out = xf * torch.rsqrt(var + eps) * weight.float()
    return out.to(x.dtype)


def fused_add_rmsnorm(
    x: torch.Tensor, residual: torch.Tensor, weight: torch.Tensor, eps: float = 1e-5
) -> Tuple[torch.Tensor, torch.Tensor]:
    """residual = residual + x (in fp32, rounded back); out = rmsnorm(residual).
    Returns (out, new_residual)."""
    new_res = (residual.float() + x.float()).to(x.dtype)
    return rmsnorm(new_res, weight, eps), new_res


# -- rotary embeddings -------------------------------------------------------

def rope_table(max_seq: int, dim: int, theta: float = 500000.0,
               device=None) -> torch.Tensor:
    """[max_seq, dim/2, 2] fp32 cos/sin table (half-split RoPE: pairs are
    (x[i], x[i + dim/2]) — Llama convention)."""
    inv = 1.0 / (theta ** (torch.arange(0, dim, 2, dtype=torch.float32,
                                        device=device) / dim))
    t = torch.arange(max_seq, dtype=torch.float32, device=device)
    freqs = torch.outer(t, inv)                      # [max_seq, dim/2]
    return torch.stack([freqs.cos(), freqs.sin()], dim=-1).contiguous()


def apply_rope(x: torch.Tensor, positions: torch.Tensor,
               table: torch.Tensor) -> torch.Tensor:
    """x: [..., S, H, D] or [..., H, D]; positions: [...,(S)] int.
    Half-split pairing: (x[:d/2], x[d/2:])."""
    D = x.shape[-1]
    cs = table[positions]                            # [..., D/2, 2]
    cos, sin = cs[..., 0], cs[..., 1]                # [..., D/2]
    cos = cos.unsqueeze(-2)                          # broadcast over heads
    sin = sin.unsqueeze(-2)
    x1 = x[..., : D // 2].float()
    x2 = x[..., D // 2:].float()
    o1 = x1 * cos - x2 * sin
    o2 = x2 * cos + x1 * sin
    return torch.cat([o1, o2], dim=-1).to(x.dtype)


def rope_kv_decode(
    q: torch.Tensor,            # [B, Hq, D] (modified logically; returns new)
    k: torch.Tensor,            # [B, Hkv, D]
    v: torch.Tensor,            # [B, Hkv, D]
    k_cache: torch.Tensor,      # [B, Hkv, max_seq, D]
    v_cache: torch.Tensor,
    pos: torch.Tensor,          # [B] int32 — write position (= current length)
    table: torch.Tensor,
) -> torch.Tensor:
    """Apply RoPE to q,k at pos; write k,v into the caches. Returns roped q."""
    q_out = apply_rope(q, pos, table)                # positions broadcast per batch
    k_rot = apply_rope(k, pos, table)
    B = q.shape[0]
    for b in range(B):
        p = int(pos[b])
        k_cache[b, :, p, :] = k_rot[b]
        v_cache[b, :, p, :] = v[b]
    return q_out


def rope_kv_prefill(
    q: torch.Tensor,            # [B, S, Hq, D]
    k: torch.Tensor,            # [B, S, Hkv, D]
    v: torch.Tensor,            # [B, S, Hkv, D]
    k_cache: torch.Tensor,
    v_cache: torch.Tensor,
    pos0: torch.Tensor,         # [B] int32 — first absolute position
    table: torch.Tensor,
) -> torch.Tensor:
    B, S = q.shape[0], q.shape[1]
    positions = pos0.view(B, 1).long() + torch.arange(S, device=q.device).view(1, S)
    q_out = apply_rope(q, positions, table)
    k_rot = apply_rope(k, positions, table)
    for b in range(B):
        p = int(pos0[b])
        k_cache[b, :, p:p + S, :] = k_rot[b].transpose(0, 1)
        v_cache[b, :, p:p + S, :] = v[b].transpose(0, 1)
    return q_out


# -- attention ---------------------------------------------------------------

def attn_decode(
    q: torch.Tensor,            # [B, Hq, D] (already roped)
    k_cache: torch.Tensor,      # [B, Hkv, max_seq, D]
    v_cache: torch.Tensor,
    seqlen: torch.Tensor,       # [B] int32 — number of valid cache entries
    scale: Optional[float] = None,
) -> torch.Tensor:
    """Single-token GQA attention over the cache. Returns [B, Hq, D]."""
    B, Hq, D = q.shape
    Hkv = k_cache.shape[1]
    G = Hq // Hkv
    scale = scale or 1.0 / math.sqrt(D)
    out = torch.empty_like(q)
    for b in range(B):
        n = int(seqlen[b])
        k = k_cache[b, :, :n, :].float()             # [Hkv, n, D]
        v = v_cache[b, :, :n, :].float()
        qb = q[b].float().view(Hkv, G, D)            # [Hkv, G, D]
        s = torch.einsum("hgd,hnd->hgn", qb, k) * scale
        p = torch.softmax(s, dim=-1)
        o = torch.einsum("hgn,hnd->hgd", p, v)
        out[b] = o.reshape(Hq, D).to(q.dtype)
    return out


def attn_prefill(
    q: torch.Tensor,            # [B, S, Hq, D] (already roped)
    k_cache: torch.Tensor,      # [B, Hkv, max_seq, D] (k/v already appended)
    v_cache: torch.Tensor,
    pos0: torch.Tensor,         # [B] int32 — q token s sits at pos0+s
    scale: Optional[float] = None,
) -> torch.Tensor:
    """Causal GQA prefill attention over the cache. q token s attends cache
    positions [0, pos0+s]. Returns [B, S, Hq, D]."""
    B, S, Hq, D = q.shape
    Hkv = k_cache.shape[1]
    G = Hq // Hkv
    scale = scale or 1.0 / math.sqrt(D)
    out = torch.empty_like(q)
    for b in range(B):
        p0 = int(pos0[b])
        n = p0 + S
        k = k_cache[b, :, :n, :].float()             # [Hkv, n, D]
        v = v_cache[b, :, :n, :].float()
        qb = q[b].float().view(S, Hkv, G, D)
        s = torch.einsum("shgd,hnd->hgsn", qb, k) * scale
        key_pos = torch.arange(n, device=q.device).view(1, 1, 1, n)
        q_pos = (p0 + torch.arange(S, device=q.device)).view(1, 1, S, 1)
        s = s.masked_fill(key_pos > q_pos, float("-inf"))
        p = torch.softmax(s, dim=-1)
        o = torch.einsum("hgsn,hnd->shgd", p, v)
        out[b] = o.reshape(S, Hq, D).to(q.dtype)
    return out


# -- encoder ops (BERT/bge architecture) --------------------------------------

def layernorm(x: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor,
              eps: float = 1e-5,
              residual: Optional[torch.Tensor] = None) -> torch.Tensor:
    """(x [+ residual]) -> LayerNorm over the last dim; f32 stats."""
    xf = x.float()
    if residual is not None:
        xf = xf + residual.float()
    mean = xf.mean(dim=-1, keepdim=True)
    var = (xf - mean).pow(2).mean(dim=-1, keepdim=True)
    out = (xf - mean) * torch.rsqrt(var + eps) * weight.float() + bias.float()
    return out.to(x.dtype)


def gelu(x: torch.Tensor) -> torch.Tensor:
    """Exact (erf) GELU."""
    return torch.nn.functional.gelu(x.float()).to(x.dtype)


# -- MLP ---------------------------------------------------------------------

def swiglu(gate_up: torch.Tensor) -> torch.Tensor:
    """gate_up: [..., 2*inter] (gate first half, up second). silu(g)*u."""
    inter = gate_up.shape[-1] // 2
    g = gate_up[..., :inter].float()
    u = gate_up[..., inter:].float()
    return (torch.nn.functional.silu(g) * u).to(gate_up.dtype)


# -- sampling ----------------------------------------------------------------

def argmax_sample(logits: torch.Tensor) -> torch.Tensor:
    """Greedy: [B, V] -> [B] int32."""
    return logits.float().argmax(dim=-1).to(torch.int32)


def gumbel_sample(logits: torch.Tensor, temperature: float,
                  generator: Optional[torch.Generator] = None) -> torch.Tensor:
    """Exact categorical sampling via the Gumbel-max trick:
    argmax(logits/T + G) with G ~ Gumbel(0,1)."""
    if temperature <= 0:
        return argmax_sample(logits)
    u = torch.rand(logits.shape, device=logits.device, dtype=torch.float32,
                   generator=generator).clamp_(1e-10, 1.0)
    g = -torch.log(-torch.log(u))
    return (logits.float() / temperature + g).argmax(dim=-1).to(torch.int32)


def topk_mask(logits: torch.Tensor, k: int) -> torch.Tensor:
    """Mask all but the top-k logits to -inf."""
    if k <= 0 or k >= logits.shape[-1]:
        return logits
    kth = torch.topk(logits.float(), k, dim=-1).values[..., -1:]
    return logits.masked_fill(logits.float() < kth, float("-inf"))


def topp_mask(logits: torch.Tensor, p: float) -> torch.Tensor:
    """Nucleus mask: keep the smallest prefix of sorted probs with mass >= p."""
    if p >= 1.0:
        return logits
    sorted_logits, idx = torch.sort(logits.float(), descending=True, dim=-1)
    probs = torch.softmax(sorted_logits, dim=-1)
    cum = probs.cumsum(dim=-1)
    keep = cum - probs < p                           # always keep the first
    masked = sorted_logits.masked_fill(~keep, float("-inf"))
    out = torch.full_like(masked, float("-inf"))
    out.scatter_(-1, idx, masked)
    return out.to(logits.dtype)


# -- fp8 weight quantization (OCP e4m3fn; decode-path serving mode) ----------

def quant_fp8(w: torch.Tensor):
    """Per-output-row absmax/448 scaling + e4m3fn encode.
    Returns (w8 uint8 [N,K], scales fp32 [N])."""
    wf = w.float()
    amax = wf.abs().amax(dim=-1).clamp_min(1e-12)
    scales = amax / 448.0
    q = (wf / scales.unsqueeze(-1)).to(torch.float8_e4m3fn)
    return q.view(torch.uint8), scales


def dequant_fp8(w8: torch.Tensor, scales: torch.Tensor) -> torch.Tensor:
    return w8.view(torch.float8_e4m3fn).float() * scales.unsqueeze(-1).float()


def hash_gumbel(B: int, v_local: int, v_offset: int, seed: int,
                step: int) -> torch.Tensor:
    """CPU replica of the GPU sampler's per-element Gumbel noise
    (fei_common.h hash_uniform: splitmix64 -> 24-bit uniform in (0,1]),
    keyed by (seed, step, batch row, GLOBAL vocab index) — so the
    tensor-parallel shard sampler matches the full sampler bit-for-bit
    in its noise stream."""
    import numpy as np

    idx = np.arange(v_offset, v_offset + v_local, dtype=np.uint64)
    out = np.empty((B, v_local), dtype=np.float32)
    with np.errstate(over="ignore"):
        for b in range(B):
            x = (np.uint64(seed)
                 ^ (np.uint64(step) * np.uint64(0x51ED27F1))
                 ^ (np.uint64(b) << np.uint64(40))
                 ^ idx)
            x = x + np.uint64(0x9E3779B97F4A7C15)
            x = (x ^ (x >> np.uint64(30))) * np.uint64(0xBF58476D1CE4E5B9)
            x = (x ^ (x >> np.uint64(27))) * np.uint64(0x94D049BB133111EB)
            x = x ^ (x >> np.uint64(31))
            m = (x >> np.uint64(40)).astype(np.float32)
            out[b] = (m + 1.0) * (1.0 / 16777216.0)
    u = torch.from_numpy(out)
    return -torch.log(-torch.log(u))


# -- ops of decoders made of unlike layers -------------------------------------
# Rows are flat [T, C]: the tokens of several sequences one after another. The
# residual, norms, angles, scores and recurrences are float32; projections and
# cached rows have the model's dtype.

def rope_table_exact(max_seq: int, dim: int, base: float,
                     device=None) -> torch.Tensor:
    """[max_seq, dim/2, 2] cos/sin of p * base^(-2i/dim), each rounded once
    from float64."""
    inv = base ** (-torch.arange(0, dim, 2, dtype=torch.float64) / max(dim, 1))
    ang = torch.outer(torch.arange(max_seq, dtype=torch.float64), inv)
    return torch.stack([ang.cos(), ang.sin()], dim=-1).float().contiguous() \
        .to(device)


def apply_rope_interleaved(x: torch.Tensor, positions: torch.Tensor,
                           table: torch.Tensor) -> torch.Tensor:
    """x [T, ..., D] float32, pairs (2i, 2i+1); positions [T]."""
    cs = table[positions.long()]
    shape = [x.shape[0]] + [1] * (x.dim() - 2) + [x.shape[-1] // 2]
    cos, sin = cs[..., 0].reshape(shape), cs[..., 1].reshape(shape)
    u, v = x[..., 0::2].float(), x[..., 1::2].float()
    return torch.stack([u * cos - v * sin, v * cos + u * sin], dim=-1) \
        .flatten(-2)


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    xf = x.float()
    return xf * torch.rsqrt(xf.pow(2).mean(dim=-1, keepdim=True) + eps)


def norm_pair(x, w1, w2, eps, dtype):
    """Two weighted RMS norms of the same rows."""
    y = rms(x, eps)
    return (y * w1).to(dtype), None if w2 is None else (y * w2).to(dtype)


def softcap_logits(y: torch.Tensor, scale: float,
                   cap: Optional[float]) -> torch.Tensor:
    y = y.float() * scale
    return y if cap is None else cap * torch.tanh(y / cap)


def latent_append(proj, m, norm_w, rot, eps, pos, dst, rows):
    """Latent (normed) and rotated key part of each row of ``proj``, into
    ``rows[dst]``; returns the rotated queries, float32 [T, H, dim+rot_dim]."""
    nq = m.heads * (m.dim + m.rot_dim)
    c = rms(proj[:, nq:nq + m.kv_rank], eps) * norm_w
    kr = proj[:, nq + m.kv_rank:nq + m.row_width].float()
    q = proj[:, :nq].float().view(-1, m.heads, m.dim + m.rot_dim).clone()
    if m.rot_dim:
        kr = apply_rope_interleaved(kr, pos, rot)
        q[..., m.dim:] = apply_rope_interleaved(
            q[..., m.dim:].contiguous(), pos, rot)
    rows[dst.long()] = torch.cat([c, kr], dim=-1).to(rows.dtype)
    return q


def latent_attend(q, pos, keys, k0, m, uk, uv, scale):
    """q [n, H, dim+rot_dim] at positions ``pos`` [n]; keys [N, row_width]
    cached rows of positions k0 .. k0+N-1. Returns [n, H, vdim]."""
    H, N = m.heads, keys.shape[0]
    c, kr = keys[:, :m.kv_rank].float(), keys[:, m.kv_rank:].float()
    k = torch.nn.functional.linear(c, uk.float()).view(N, H, m.dim)
    v = torch.nn.functional.linear(c, uv.float()).view(N, H, m.vdim)
    s = torch.einsum("nhd,khd->hnk", q[..., :m.dim], k)
    if m.rot_dim:
        s = s + torch.einsum("nhd,kd->hnk", q[..., m.dim:], kr)
    s = s * scale
    kp = torch.arange(k0, k0 + N, device=q.device).view(1, 1, N)
    qp = pos.long().view(1, -1, 1)
    hide = kp > qp
    if m.window is not None:
        hide = hide | (qp - kp >= m.window)
    p = torch.softmax(s.masked_fill(hide, float("-inf")), dim=-1)
    return torch.einsum("hnk,khd->nhd", p, v)


def gla_log_decay(a1, a2, bias, tau):
    """log of sigmoid(z)^(1/tau), z = a2 a1 + bias; float32 [T, H*dim]."""
    z = torch.nn.functional.linear(a1.float(), a2.float()) + bias
    return torch.nn.functional.logsigmoid(z) / tau


def gla_scan(q, k, v, logdecay, state):
    """q, k, logdecay [T, H, d], v [T, H, e], state [H, e, d] (float32),
    token by token. Returns o [T, H, e] and the last state."""
    out = torch.empty(q.shape[0], q.shape[1], v.shape[-1])
    S = state.clone()
    decay = logdecay.exp()
    for t in range(q.shape[0]):
        S = S * decay[t].unsqueeze(1) + v[t].unsqueeze(-1) * k[t].unsqueeze(1)
        out[t] = (S * q[t].unsqueeze(1)).sum(-1)
    return out, S


def gla_gate_out(o, g, norm_w, eps):
    """Per-head RMS norm of o [T, H, e], times silu(g) [T, H*e]."""
    y = (rms(o, eps) * norm_w).flatten(1)
    gf = g.float()
    return y * (gf * torch.sigmoid(gf))


def short_conv(u, first, weights):
    """u [n, channels] float32, the ``taps - 1`` projections before it in
    ``first`` (zeros before the sequence's start), weights [taps, channels]."""
    taps = weights.shape[0]
    ext = torch.cat([first, u])
    y = torch.zeros_like(u)
    for j in range(taps):
        y = y + weights[j] * ext[j:j + u.shape[0]]
    return y


def sigmoid_attend(q, pos, keys, k0, m, bias):
    """q [n, H, dim] at positions ``pos`` [n]; keys [N, row_width] cached rows
    of positions k0 .. k0+N-1; bias [3, H]: r1, r2, pb. Returns [n, H, vdim]."""
    N, G = keys.shape[0], m.kv_heads
    k = keys[:, :G * m.dim].float().view(N, G, m.dim)
    v = keys[:, G * m.dim:].float().view(N, G, m.vdim)
    k, v = (t.repeat_interleave(m.heads // G, dim=1) for t in (k, v))
    s = torch.einsum("nhd,khd->hnk", q, k) * m.scale
    d = pos.long().view(-1, 1) - torch.arange(k0, k0 + N).view(1, -1)
    r1, r2, pb = (b.view(-1, 1, 1) for b in bias)
    s = s - r1 * torch.log(1.0 + r2 * d.clamp(min=0).float()) + pb
    hide = d < 0
    if m.window is not None:
        hide = hide | (d >= m.window)
    w = torch.sigmoid(s).masked_fill(hide, 0.0)
    return torch.einsum("hnk,khd->nhd", w, v)


def square_relu(x):
    return torch.relu(x.float()).square()


def route(logits, top, scale):
    """Sigmoid router: (experts [T, top], weights [T, top] float32)."""
    s = torch.sigmoid(logits.float())
    ids = torch.topk(logits.float(), top, dim=-1).indices
    w = s.gather(1, ids)
    return ids, w / (w.sum(-1, keepdim=True) + 1e-20) * scale


def moe(h, ids, weights, up, down):
    """sum_k weights[t, k] * down[e] relu(up[e] h[t])^2, e = ids[t, k];
    float32."""
    out = torch.zeros(h.shape[0], down.shape[1])
    for e in range(up.shape[0]):
        t, k = (ids == e).nonzero(as_tuple=True)
        if t.numel():
            a = square_relu(torch.nn.functional.linear(h[t], up[e]))
            y = torch.nn.functional.linear(a.to(h.dtype), down[e]).float()
            out.index_add_(0, t, y * weights[t, k].unsqueeze(1))
    return out
