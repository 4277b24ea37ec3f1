"""Bokenex against a plain implementation (tests/bokenex_oracle.py): every
mechanism alone, prompts, decoding, portions, mixed batches, reuse of blocks
and slots, window edges, generation through the engine and the sessions.

Each test runs on the CPU reference ops, and on the GPU with the HIP kernels.
"""

import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import bokenex_oracle as oracle
import step_helpers
from fei_amd import ops
from fei_amd.engine.config import (MODEL_SPECS, BokenexSpec, MoESpec,
                                   get_spec)
from fei_amd.engine.step import StepEntry
from fei_amd.models.bokenex import BokenexModel
from step_helpers import (DEVICES, F32_TOL, err, row_errors, run, run_mixed,
                          serve_sessions, toks)

DTYPES = [torch.float32, torch.bfloat16]


def att(heads=4, kv_heads=2, dim=20, vdim=28, window=37, conv=3, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
         "scale": scale or dim ** -0.5, "conv": conv}
    if window:
        m["mask"] = {"size": window}
    return m


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, scale=1.5):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top, "scale": scale}}


def make_cfg(layers, width=52, vocab=101, mult=0.6, positions=512, eps=3e-5):
    """layers: (mixer, feed-forward or None) each."""
    return {"architecture": "Bokenex", "vocab": vocab, "width": width,
            "max_positions": positions, "residual_mult": mult,
            "norm": {"eps": eps},
            "layers": [{"type": "attention", "mixer": m, "mlp": f}
                       for m, f in layers]}


CONFIGS = {
    # no size a multiple of 8, unlike layers, one without a feed-forward
    "odd": make_cfg([(att(), dense(36)), (att(6, 3, 9, 14, 70, 5), None),
                     (att(3, 3, 17, 11, 50, 2), moe(5, 2, 21)),
                     (att(5, 1, 12, 30, 9, 4), moe(3, 3, 10, 0.7))]),
    # multiples of 8 (vector paths), more than 16 heads on a key head
    "even": make_cfg([(att(18, 1, 32, 40, 72, 4), moe(8, 3, 48)),
                      (att(8, 4, 24, 16, 64, 3), dense(96))], width=64,
                     vocab=96),
    # no window, no convolution, one expert, one head
    "full": make_cfg([(att(1, 1, 40, 56, None, 1), moe(1, 1, 40)),
                      (att(2, 2, 64, 128, None, 4), dense(40))], width=48,
                     vocab=77, mult=1.0),
}


def Net(tmp, cfg, seed=0, device="cpu", dtype=torch.float32, edit=None,
        max_seq=512):
    return step_helpers.Net(tmp, oracle, cfg, seed, device, dtype, edit,
                            max_seq)


# -- mechanisms alone ------------------------------------------------------------

@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_every_layer(tmp_path, name, device):
    """The residual after each layer: both sublayers, norm, positions."""
    net = Net(tmp_path, CONFIGS[name], 1, device)
    tokens = toks(70, net.cfg["vocab"], 2)
    keep, got = [], []
    oracle.forward(tokens, net.W, net.cfg, keep)
    r = net.runner()
    batch = r.build([StepEntry(r.admit(), tokens, [0])])
    with torch.no_grad():
        net.model.forward(batch, r.cache, lambda i, x: got.append(x.clone()))
    assert len(got) == len(keep)
    for a, b in zip(got, keep):
        assert err(a, b) < F32_TOL


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ids", [torch.int32, torch.int64])
def test_embedding_and_positions(device, dtype, ids):
    g = torch.Generator().manual_seed(1)
    emb, pos_emb = (torch.randn(n, 300, generator=g).to(dtype)
                    for n in (50, 40))
    tok = torch.randint(0, 50, (33,), generator=g)
    pos = torch.randint(0, 40, (33,), generator=g)
    x = ops.embed_pos(tok.to(device, ids), pos.to(device, torch.int32),
                      emb.to(device), pos_emb.to(device))
    assert x.dtype == torch.float32
    assert torch.equal(x.cpu(), emb[tok].float() + pos_emb[pos].float())


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 6])
def test_attention_alone(tmp_path, taps, device):
    """One layer without a feed-forward, whatever the convolution's length,
    from prompts, in portions shorter than it, and token by token."""
    cfg = make_cfg([(att(conv=taps), None)])
    net = Net(tmp_path, cfg, 3, device)
    tokens = toks(110, cfg["vocab"], 4)
    want = net.want(tokens)
    r = net.runner(slots=1)
    for sizes in ([110], [1], [2], [1, 2, 3, 1, 50]):
        sid = r.admit()
        assert err(run(r, sid, tokens, sizes), want) < F32_TOL, sizes
        r.release(sid)


@pytest.mark.parametrize("device", DEVICES)
def test_convolution_sees_its_taps_only(tmp_path, device):
    """A window of one key: the output depends on the token and the taps - 1
    before it, each of them, and on nothing else."""
    taps = 4
    cfg = make_cfg([(att(2, 1, 16, 16, 1, taps), None)], width=32)

    def edit(W):
        W["l0.mix.v"] *= 8.0
        W["l0.mix.pb"] += 4.0
    net = Net(tmp_path, cfg, 5, device, edit=edit)
    a = toks(80, cfg["vocab"], 6)
    r = net.runner(slots=1)

    def last(tokens, sizes):
        sid = r.admit()
        out = run(r, sid, tokens, sizes)[-1]
        r.release(sid)
        return out.double().cpu()
    for sizes in ([80], [64, 15, 1], [77, 3], [78, 1], [76, 2]):
        base = last(a, sizes)
        for back in range(1, taps + 2):
            b = list(a)
            b[-1 - back] = (b[-1 - back] + 7) % cfg["vocab"]
            moved = float((last(b, sizes) - base).norm() / base.norm())
            assert moved > 1e-3 if back < taps else moved == 0.0, (sizes, back)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("r1,r2", [(0.0, 1.0), (3.0, 0.01), (0.2, 40.0),
                                   (12.0, 2.0)])
def test_distance_bias(tmp_path, device, r1, r2):
    """From none to one that leaves little but the token itself."""
    cfg = make_cfg([(att(window=None, conv=1), None)])

    def edit(W):
        W["l0.mix.r1"][:] = r1
        W["l0.mix.r2"][:] = r2
        W["l0.mix.r1"][1] = 0.5                  # heads differ
        W["l0.mix.pb"] += 3.0
    net = Net(tmp_path, cfg, 7, device, edit=edit)
    tokens = toks(200, cfg["vocab"], 8)
    want = net.want(tokens)
    r = net.runner()
    assert err(run(r, r.admit(), tokens, [200]), want) < F32_TOL
    assert err(run(r, r.admit(), tokens, [150, 1, 1]), want) < F32_TOL


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("shift", [-60.0, -12.0, 9.0, 60.0])
def test_weights_from_none_to_all(tmp_path, device, shift):
    """Sigmoids from e^-60 to 1: nothing is normalized, nothing overflows."""
    cfg = make_cfg([(att(scale=3.0), None)])

    def edit(W):
        W["l0.mix.pb"] += shift
    net = Net(tmp_path, cfg, 9, device, edit=edit)
    tokens = toks(100, cfg["vocab"], 10)
    want = net.want(tokens)
    r = net.runner()
    assert err(run(r, r.admit(), tokens, [90, 1]), want) < F32_TOL


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("experts,top", [(1, 1), (4, 4), (7, 2), (64, 8),
                                         (130, 5), (1000, 3)])
def test_router(device, experts, top):
    g = torch.Generator().manual_seed(experts)
    z = torch.randn(37, experts, generator=g) * 4.0
    z[3] += 30.0                       # scores that all round to 1
    z[4] -= 60.0                       # and to almost nothing
    ids, w = ops.route(z.to(device), top, 1.7)
    for t in range(z.shape[0]):
        want = oracle.route(z[t].double(), top, 1.7)
        if t != 3:                     # there the oracle's scores are equal
            assert sorted(ids[t].tolist()) == sorted(e for e, _ in want)
        want = dict(want) if t != 3 else dict.fromkeys(ids[t].tolist(),
                                                       1.7 / top)
        for e, x in zip(ids[t].tolist(), w[t].tolist()):
            assert abs(x - want[e]) < 1e-5


@pytest.mark.gpu
def test_router_without_numbers():
    """Logits that are not numbers still choose experts that exist."""
    z = torch.full((3, 6), float("nan"), device="cuda")
    z[1, 4] = 1.0
    ids, _ = ops.route(z, 3, 1.0)
    assert int(ids.min()) >= 0 and int(ids.max()) < 6


def experts_want(x, gain, eps, a, w_o, up, down, router, f, mult):
    """Oracle of residual_moe, float64."""
    W = {"router": router}
    for e in range(up.shape[0]):
        W[f"e{e}.up"], W[f"e{e}.down"] = up[e], down[e]
    h = oracle.rms_norm(x, gain, eps)
    mlp = moe(f.experts, f.top, f.ff, f.scale)
    return x + mult * (a @ w_o.T + oracle.experts(h, W, "", mlp))


# experts, top, their width, width: scalar sizes, sizes of the skinny and of
# the tiled products, more experts than rows
MOE_SIZES = [(5, 2, 21, 52), (6, 3, 64, 128), (4, 2, 192, 1024),
             (40, 4, 72, 64), (3, 1, 128, 320), (2, 2, 640, 192)]


MOE_CASES = [("cpu", torch.float32, n) for n in (1, 9)] + [
    pytest.param("cuda", dtype, n, marks=pytest.mark.gpu)
    for dtype in DTYPES for n in (1, 2, 3, 4, 8, 9, 100, 300)]


@pytest.mark.parametrize("size", MOE_SIZES)
@pytest.mark.parametrize("device,dtype,rows", MOE_CASES)
def test_experts(device, dtype, rows, size):
    """Every route of a mixture layer's products: skinny, small and large
    tiles; rows that crowd one expert and experts without any row."""
    E, top, ff, C = size
    f = MoESpec(E, top, ff, 1.3)
    g = torch.Generator().manual_seed(rows + C)
    rand = lambda *s: torch.randn(*s, generator=g).bfloat16().float()
    x, n_o = rand(rows, C), 40
    x[rows // 2:, :] = x[rows // 2, :] + 0.01 * x[rows // 2:, :]   # crowd
    x = x.bfloat16().float()
    router = rand(E, C) * (4.0 / C ** 0.5)
    up = (rand(E, ff, C) / C ** 0.5).bfloat16().float()
    down = (rand(E, C, ff) / ff ** 0.5).bfloat16().float()
    w_o = (rand(C, n_o) / n_o ** 0.5).bfloat16().float()
    router = router.bfloat16().float()
    gain, eps, mult = torch.tensor(1.25), 1e-4, 0.4
    a = rand(rows, n_o)
    dev = lambda t: t.to(device, dtype)
    norm = ops.GainNorm(gain.to(device), C, eps)
    h = ops.GainNormed(x.to(device), norm, dtype)
    empty = torch.empty(rows, 0, dtype=dtype, device=device)
    w_in = torch.cat([rand(16, C), router])
    proj, z = ops.parallel_in(h, dev(w_in), 16, 0, E, empty)
    d = lambda t: t.double()
    hw = oracle.rms_norm(d(x), 1.25, eps)
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    assert z.dtype == torch.float32
    assert err(z.view(1, -1), (hw @ d(router).T).view(1, -1)) < tol
    assert err(proj, hw @ d(w_in[:16]).T) < tol
    # the exact choice, so that no close call decides
    z = (hw @ d(router).T).float().to(device)
    got = ops.residual_moe(x.to(device), h, z, dev(a), dev(w_o), dev(up),
                           dev(down), f, mult)
    want = experts_want(d(x), 1.25, eps, d(a), d(w_o), d(up), d(down),
                        d(router), f, mult)
    assert err(got - x.to(device), want - d(x)) < (
        2e-5 if dtype == torch.float32 else 1.2e-2)


@pytest.mark.gpu
@pytest.mark.parametrize("size", [(8, 2, 1536, 1536), (3, 2, 64, 3072)])
def test_many_experts_rows(size):
    """Enough tiles for the widest blocks of the grouped product, the last of
    each expert not full."""
    E, top, ff, C = size
    T = 4001
    g = torch.Generator(device="cuda").manual_seed(T)
    rand = lambda *s: torch.randn(*s, generator=g, device="cuda")
    x = rand(T, C)
    up, down = ((rand(E, *s) / s[1] ** 0.5).bfloat16()
                for s in ((ff, C), (C, ff)))
    z = rand(T, E) * 3.0
    w_o, a = torch.zeros(C, 8, device="cuda").bfloat16(), \
        torch.zeros(T, 8, device="cuda").bfloat16()
    norm = ops.GainNorm(torch.ones((), device="cuda"), C, 1e-5)
    h = ops.GainNormed(x, norm, torch.bfloat16)
    rows = h.rows.clone()
    f = MoESpec(E, top, ff, 1.0)
    got = ops.residual_moe(torch.zeros_like(x), h, z, a, w_o, up, down, f, 1.0)
    ids, w = ops.ref.route(z.cpu(), top, 1.0)
    some = torch.randperm(T, generator=torch.Generator().manual_seed(1))[:64]
    want = ops.ref.moe(rows[some].float().cpu(), ids[some], w[some],
                       up.float().cpu(), down.float().cpu())
    assert err(got[some], want) < 1.2e-2
    assert bool(torch.isfinite(got).all())


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 2, 3, 4, 7, 8, 9, 33])
@pytest.mark.parametrize("width,n_mix,ff", [(1024, 96, 64), (2048, 144, 9000),
                                            (88, 31, 40), (52, 7, 21),
                                            (64, 10, 0)])
def test_products(rows, width, n_mix, ff, dtype):
    """Every route of a parallel layer's products against float64 on the same
    values: norm inside, matrix tile, library."""
    g = torch.Generator().manual_seed(rows + width)
    bf = lambda *s: torch.randn(*s, generator=g).bfloat16()
    x = torch.randn(rows, width, generator=g) * 3.0
    w_in = bf(n_mix + ff, width) / width ** 0.5
    d = lambda t: t.double()
    norm = ops.GainNorm(torch.tensor(0.8, device="cuda"), width, 1e-3)
    cat = torch.zeros(rows, n_mix + ff, dtype=dtype, device="cuda")
    h = ops.GainNormed(x.cuda(), norm, dtype)
    proj, router = ops.parallel_in(h, w_in.to("cuda", dtype), n_mix, ff, 0,
                                   cat[:, n_mix:])
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    want = oracle.rms_norm(d(x), 0.8, 1e-3) @ d(w_in).T
    assert router is None
    assert err(proj, want[:, :n_mix]) < tol
    if ff:
        assert err(cat[:, n_mix:], oracle.square_relu(want[:, n_mix:])) < \
            2 * tol
        assert not cat[:, :n_mix].any()
    w = bf(n_mix + 50, width) / width ** 0.5
    y = ops.gain_logits(h, w.to("cuda", dtype))
    assert err(y, oracle.rms_norm(d(x), 0.8, 1e-3) @ d(w).T) < tol
    res, a = torch.randn(rows, n_mix + 50, generator=g), bf(rows, width)
    y = ops.residual_linear(res.cuda(), a.to("cuda", dtype),
                            w.to("cuda", dtype), 0.3)
    assert err(y, d(res) + 0.3 * d(a) @ d(w).T) < 1e-5


# -- prompts, decoding, portions ---------------------------------------------------

@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_prompt_decode_and_portions_agree(tmp_path, name, device):
    net = Net(tmp_path, CONFIGS[name], 11, device)
    tokens = toks(141, net.cfg["vocab"], 12)
    want = net.want(tokens)
    r = net.runner(slots=1)
    for sizes in ([141], [1], [2], [64], [63, 65], [2, 3, 5, 7, 1, 31],
                  [90, 1, 1, 2], [128, 1]):
        sid = r.admit()
        assert err(run(r, sid, tokens, sizes), want) < F32_TOL, sizes
        r.release(sid)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("block_size", [8, 16, 32, 128])
def test_block_sizes(tmp_path, block_size, device):
    """Blocks smaller than the kernels' key tiles, and larger."""
    net = Net(tmp_path, CONFIGS["even"], 13, device)
    tokens = toks(141, net.cfg["vocab"], 14)
    want = net.want(tokens)
    r = net.runner(blocks=256 // block_size, slots=1, block_size=block_size)
    for sizes in ([141], [100, 1], [33, 1, 7]):
        sid = r.admit()
        assert err(run(r, sid, tokens, sizes), want) < F32_TOL, sizes
        r.release(sid)


@pytest.mark.gpu
@pytest.mark.parametrize("name", list(CONFIGS))
def test_bfloat16(tmp_path, name):
    """Rounding turns a close choice of experts now and then, which changes a
    row by much more than rounding: a few rows may be off."""
    net = Net(tmp_path, CONFIGS[name], 11, "cuda", torch.bfloat16)
    tokens = toks(141, net.cfg["vocab"], 12)
    want = net.want(tokens)
    r = net.runner(slots=1)
    for sizes in ([141], [1], [2, 3, 61, 1]):
        sid = r.admit()
        e = row_errors(run(r, sid, tokens, sizes), want)
        assert float(e.quantile(0.9)) < 0.03, (sizes, e.sort().values[-20:])
        assert float(e.max()) < 0.6, sizes
        r.release(sid)


@pytest.mark.parametrize("device", DEVICES)
def test_first_tokens(tmp_path, device):
    net = Net(tmp_path, CONFIGS["odd"], 15, device)
    r = net.runner()
    for n in (1, 2, 3, 4, 5, 6):
        tokens = toks(n, net.cfg["vocab"], 20 + n)
        for sizes in ([n], [1], [2]):
            sid = r.admit()
            assert err(run(r, sid, tokens, sizes), net.want(tokens)) < F32_TOL
            r.release(sid)


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding(tmp_path, device):
    """Decoding past several windows and blocks."""
    net = Net(tmp_path, CONFIGS["odd"], 16, device)
    tokens = toks(330, net.cfg["vocab"], 17)
    r = net.runner()
    got = run(r, r.admit(), tokens, [30] + [1] * 300)
    assert err(got, net.want(tokens)) < F32_TOL


SIZES = {
    # the sizes of a real model's layers
    "usual": [att(32, 8, 128, 128, 100, 4), att(32, 8, 64, 64, 90, 4)],
    # the largest head sizes the kernels take
    "largest": [att(2, 1, 256, 256, 70, 4), att(4, 2, 192, 224, 130, 3)],
    # between the sizes that kernels are built for, vector paths
    "between": [att(20, 1, 72, 88, 90, 5), att(6, 2, 136, 40, 300, 2)],
    # the same without them
    "ragged": [att(5, 5, 67, 85, 90, 3), att(34, 2, 131, 21, 65, 4)],
}


@pytest.mark.gpu
@pytest.mark.parametrize("name", list(SIZES))
@pytest.mark.parametrize("dtype", DTYPES)
def test_other_sizes(tmp_path, name, dtype):
    cfg = make_cfg([(m, None) for m in SIZES[name]], width=64, vocab=40)
    net = Net(tmp_path, cfg, 60, "cuda", dtype)
    tokens = toks(140, 40, 61)
    want = net.want(tokens)
    r = net.runner(slots=1)
    tol = F32_TOL if dtype == torch.float32 else 0.03
    for sizes in ([140], [131, 1], [5, 66, 1]):
        sid = r.admit()
        assert err(run(r, sid, tokens, sizes), want) < tol, sizes
        r.release(sid)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [None, 1000])
def test_many_splits(tmp_path, dtype, window):
    """A long context: a decode row's keys in many splits, batched rows of
    unlike lengths, tiles past the first block of queries."""
    cfg = make_cfg([(att(4, 2, 32, 32, window, 4), None)], width=32, vocab=40,
                   positions=2048)

    def edit(W):
        W["l0.mix.r1"] *= 0.1            # far keys keep their weight
    net = Net(tmp_path, cfg, 62, "cuda", dtype, edit=edit, max_seq=2048)
    tokens = toks(1400, 40, 63)
    want = net.want(tokens)
    r = net.runner(blocks=64)
    tol = F32_TOL if dtype == torch.float32 else 0.02
    assert err(run(r, r.admit(), tokens, [1370, 1, 1, 28]), want) < tol
    sids = [r.admit() for _ in range(3)]
    lens = (1399, 130, 1)
    r.step([StepEntry(s, tokens[:n]) for s, n in zip(sids, lens)])
    got = r.step([StepEntry(s, [tokens[n]], [0]) for s, n in zip(sids, lens)])
    assert err(got, want[list(lens)]) < tol


# -- window edges -------------------------------------------------------------------

def every_key_counts(W):
    """No distance bias, even weights, values that outweigh the residual: no
    key of a window is without weight."""
    W["l0.mix.r1"] *= 0.0
    W["l0.mix.q.norm"] *= 0.2
    W["l0.mix.v"] *= 6.0
    W["pos"] *= 0.1


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("conv", [1, 3])
@pytest.mark.parametrize("window", [1, 2, 31, 32, 33, 63, 64, 65, 100, 128])
def test_window_edge(tmp_path, window, conv, device):
    """Changing the first token that a query's window reaches (through the
    convolution of the window's first key) changes the output of one
    attention layer; the token before it changes nothing. In a prompt, in
    portions and in decoding, with queries around block borders."""
    cfg = make_cfg([(att(2, 1, 16, 16, window, conv), None)], width=32,
                   vocab=71, mult=1.0)
    net = Net(tmp_path, cfg, 18, device, edit=every_key_counts)
    a = toks(200, cfg["vocab"], 19)
    r = net.runner(slots=1)

    def logits(tokens, sizes):
        sid = r.admit()
        out = run(r, sid, tokens, sizes)
        r.release(sid)
        return out

    schedules = ([200], [70, 1, 1, 40, 2], [1])
    want = net.want(a)
    for s in schedules:
        assert err(logits(a, s), want) < F32_TOL, s
    for q in (127, 128, 192, 199):
        for inside in (True, False):
            k = q - window + 1 - (conv - 1) - (0 if inside else 1)
            if k < 0 or k == q:
                continue
            # of some tokens at place k, the one that moves the output most
            moved, b, new = max(
                (((y - want[q]).norm() / want[q].norm()).item(), c, y)
                for c, y in ((c, net.want(c)[q]) for c in (
                    a[:k] + [(a[k] + d) % cfg["vocab"]] + a[k + 1:q + 1]
                    for d in (7, 19))))
            assert moved > 20 * F32_TOL if inside else moved < 1e-12
            for s in schedules:
                assert err(logits(b, s)[q][None], new[None]) < F32_TOL, (q, s)


@pytest.mark.gpu
@pytest.mark.parametrize("window", [1, 31, 32, 33, 64, 100])
def test_window_edge_in_bfloat16(tmp_path, window):
    """The token before the first that a window reaches does not change a bit
    of the logits; the first one does, as much as it should."""
    conv = 2
    cfg = make_cfg([(att(4, 1, 64, 64, window, conv), None)], width=32,
                   vocab=71, mult=1.0)
    net = Net(tmp_path, cfg, 20, "cuda", torch.bfloat16, edit=every_key_counts)
    r = net.runner(slots=1)

    def logits(tokens, sizes):
        sid = r.admit()
        out = run(r, sid, tokens, sizes)
        r.release(sid)
        return out
    a = toks(200, cfg["vocab"], 19)
    for q in (127, 128, 199):
        k = q - window + 1 - (conv - 1)
        b, c = list(a), list(a)
        b[k] = (b[k] + 7) % cfg["vocab"]
        c[k - 1] = (c[k - 1] + 7) % cfg["vocab"]
        want = net.want(b)[q] - net.want(a)[q]
        for s in ([200], [70, 1, 1, 40, 2], [1]):
            base = logits(a, s)[q]
            assert torch.equal(logits(c, s)[q], base), (q, s)
            moved = (logits(b, s)[q] - base).double().cpu()
            assert float((moved - want).norm()) < 0.35 * float(want.norm())


@pytest.mark.parametrize("device", DEVICES)
def test_far_key_among_many(tmp_path, device):
    """One key far back that stands out from hundreds of others, at block and
    tile borders: its token alone has a query-like key, and its weight is near
    one where the others' are near nothing."""
    cfg = make_cfg([(att(1, 1, 16, 24, None, 1, scale=1.5), None)], width=32)
    mark = cfg["vocab"] - 1

    def edit(W):
        W["pos"] *= 0.0
        W["l0.mix.r1"][:] = 0.3
        W["l0.mix.pb"][:] = -18.0
        for n in ("", ".conv", ".norm"):
            W["l0.mix.k" + n][:] = W["l0.mix.q" + n]
        W["l0.mix.q.norm"][:] = W["l0.mix.k.norm"][:] = 1.0
        # every token but the marked one turns away from its direction
        e = W["embed"][mark] / W["embed"][mark].norm()
        W["embed"] -= torch.outer(W["embed"] @ e, e)
        W["embed"][mark] = 9.0 * e
    net = Net(tmp_path, cfg, 21, device, edit=edit)
    r = net.runner(slots=1)
    for k in (0, 1, 31, 32, 63, 64, 127, 128):
        tokens = toks(260, mark, 22)
        tokens[k] = tokens[-1] = tokens[210] = mark
        want = net.want(tokens)
        other = list(tokens)
        other[k] = 5
        assert err(net.want(other)[-1:], want[-1:]) > 0.02
        for sizes in ([260], [200, 1, 1, 30, 27, 1]):
            sid = r.admit()
            assert err(run(r, sid, tokens, sizes), want) < 1e-4, (k, sizes)
            r.release(sid)


# -- batches, blocks and slots ---------------------------------------------------------

@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", ["odd", "even"])
def test_mixed_batches(tmp_path, name, device):
    """Unequal requests in one batch, portions beside single tokens, requests
    that pause, end and make room for others."""
    net = Net(tmp_path, CONFIGS[name], 23, device)
    reqs = {i: toks(n, net.cfg["vocab"], 30 + i)
            for i, n in enumerate((150, 97, 64, 33, 120))}
    r = net.runner(blocks=8, slots=3)
    got = run_mixed(r, reqs)
    for i, t in reqs.items():
        assert err(got[i], net.want(t)) < F32_TOL, i
    assert r.cache.free_blocks() == 8 and r.cache.free_slots() == 3


@pytest.mark.parametrize("device", DEVICES)
def test_decode_batches(tmp_path, device):
    """Single tokens of 1 to 9 sequences of unlike lengths, each as alone."""
    net = Net(tmp_path, CONFIGS["even"], 24, device)
    V = net.cfg["vocab"]
    seqs = [toks(n, V, 50 + n) for n in (3, 90, 64, 1, 41, 128, 7, 65, 20)]
    want = [net.want(t)[-1] for t in seqs]
    for n in (1, 2, 3, 4, 8, 9):
        r = net.runner(blocks=20, slots=9)
        sids = [r.admit() for _ in range(n)]
        first = [StepEntry(s, t[:-1]) for s, t in zip(sids, seqs) if t[:-1]]
        if first:
            r.step(first)
        got = r.step([StepEntry(s, t[-1:], [0]) for s, t in zip(sids, seqs)])
        assert err(got, torch.stack(want[:n])) < F32_TOL, n


@pytest.mark.parametrize("device", DEVICES)
def test_wanted_rows_follow_the_entries(tmp_path, device):
    """Logits come in the order of the entries although single tokens are
    packed first."""
    net = Net(tmp_path, CONFIGS["even"], 25, device)
    V = net.cfg["vocab"]
    a, b, c = toks(20, V, 1), toks(9, V, 2), toks(12, V, 3)
    r = net.runner()
    sa, sb, sc = r.admit(), r.admit(), r.admit()
    r.step([StepEntry(sb, b[:8])])
    got = r.step([StepEntry(sa, a, [3, 19]), StepEntry(sb, b[8:], [0]),
                  StepEntry(sc, c, [0])])
    want = torch.stack([net.want(a)[3], net.want(a)[19], net.want(b)[8],
                        net.want(c)[0]])
    assert err(got, want) < F32_TOL
    # a step that asks for nothing
    assert r.step([StepEntry(sa, [1, 2]), StepEntry(sc, [3])]).shape == (0, V)


@pytest.mark.parametrize("device", DEVICES)
def test_blocks_and_slots_used_again(tmp_path, device):
    """Sequences one after another on the same blocks and slot."""
    net = Net(tmp_path, CONFIGS["odd"], 26, device)
    V = net.cfg["vocab"]
    r = net.runner(blocks=2, slots=1)
    for seed, sizes in ((1, [100]), (2, [1]), (3, [7, 64]), (4, [90, 1]),
                        (5, [1, 2])):
        tokens = toks(100, V, seed)
        sid = r.admit()
        assert err(run(r, sid, tokens, sizes), net.want(tokens)) < F32_TOL
        with pytest.raises(MemoryError):
            r.admit()
        r.release(sid)


@pytest.mark.parametrize("device", DEVICES)
def test_fork(tmp_path, device):
    """A copy goes on by itself: rows and state are its own."""
    net = Net(tmp_path, CONFIGS["even"], 27, device)
    V = net.cfg["vocab"]
    a = toks(70, V, 1)
    b = a[:50] + toks(20, V, 2)
    r = net.runner()
    sa = r.admit()
    run(r, sa, a[:50], [50])
    sb = r.cache.fork(sa)
    r.set_length(sb, 50)
    for sid, t in ((sa, a), (sb, b)):
        assert err(run(r, sid, t[50:], [1, 3]), net.want(t)[50:]) < F32_TOL


# -- configuration and weights ------------------------------------------------------

def test_config_round_trip(tmp_path):
    net = Net(tmp_path / "a", CONFIGS["odd"], 28)
    net.model.save_weights(str(tmp_path / "b"))
    spec = get_spec(str(tmp_path / "b"))
    assert spec.layers == net.model.spec.layers
    again = BokenexModel(spec, torch.device("cpu"), torch.float32,
                         weights=str(tmp_path / "b"))
    out = again.state_dict_full()
    assert set(out) == set(net.W)
    for k, v in net.model.state_dict_full().items():
        assert torch.equal(v, out[k]), k
        assert torch.equal(v.double(), net.W[k]), k


def test_unknown_config_is_refused():
    for path, value in ((("layers", 0, "mixer", "bias"), True),
                        (("layers", 0, "type"), "gla"),
                        (("layers", 0, "mlp", "kind"), "other"),
                        (("layers", 2, "mlp", "router", "groups"), 2),
                        (("layers", 2, "mlp", "router", "top"), 6),
                        (("layers", 0, "mixer", "kv_heads"), 3),
                        (("layers", 0, "mixer", "mask", "size"), 0),
                        (("layers", 0, "mixer", "mask", "chunk"), 8),
                        (("extra",), 1)):
        cfg = json.loads(json.dumps(CONFIGS["odd"]))
        d = cfg
        for k in path[:-1]:
            d = d[k]
        d[path[-1]] = value
        with pytest.raises(ValueError):
            BokenexSpec.from_config(cfg, {})


def test_wrong_tensors_are_refused(tmp_path):
    from safetensors.torch import load_file, save_file
    net = Net(tmp_path, CONFIGS["odd"], 29)
    f = os.path.join(net.path, "model.safetensors")
    full = load_file(f)
    missing = {k: v for k, v in full.items() if k != "l2.mlp.e1.up"}
    extra = dict(full, other=torch.zeros(1))
    shape = dict(full, **{"l0.norm1": torch.zeros(52)})
    for bad in (missing, extra, shape):
        save_file(bad, f)
        with pytest.raises(ValueError):
            BokenexModel(net.model.spec, torch.device("cpu"), torch.float32,
                         weights=net.path)


def test_no_position_past_the_last(tmp_path):
    cfg = make_cfg([(att(), None)], positions=40)
    net = Net(tmp_path, cfg, 31, max_seq=40)
    r = net.runner()
    tokens = toks(40, cfg["vocab"], 1)
    s = r.admit()
    assert err(run(r, s, tokens, [40]), net.want(tokens)) < F32_TOL
    with pytest.raises(ValueError):
        r.step([StepEntry(s, [1])])
    with pytest.raises(ValueError):
        net.model.resize(41)


def test_sizes_the_kernels_do_not_take():
    with pytest.raises(ValueError):
        spec = BokenexSpec.from_config(
            make_cfg([(att(dim=300), None)]), {})
        BokenexModel(spec, torch.device("cpu"), torch.float32)


def test_registered_specs():
    for name, spec in MODEL_SPECS.items():
        if spec.arch == "bokenex":
            assert spec.params_bytes() > 0 and get_spec(name) is spec
            assert BokenexSpec.from_config(
                spec.to_config(), {}, name).layers == spec.layers
    for size in ("1b", "8b"):
        a, b = (MODEL_SPECS[f"{n}-{size}"].params_bytes()
                for n in ("bokenex", "llama3"))
        assert abs(a / b - 1) < 0.05
    m = BokenexModel(get_spec("bokenex-tiny"), torch.device("cpu"),
                     torch.float32, seed=3)
    assert m.param_bytes() == 4 * sum(
        t.numel() for t in m.state_dict_full().values()) == \
        m.spec.params_bytes(4)
    assert m.cache_bytes_per_token() == 4 * 4 * 2 * (24 + 40)


# -- generation ----------------------------------------------------------------------

GEN = make_cfg([(att(4, 2, 16, 24, 30, 4), moe(4, 2, 24)),
                (att(2, 1, 24, 16, 45, 3), dense(48))], width=64, vocab=272,
               positions=256)


def sharp(W):
    """Logits far enough apart that rounding does not change the largest."""
    W["head"] *= 3.0


def engine_for(tmp_path, device, **kw):
    from fei_amd.engine.engine import LocalEngine
    net = Net(tmp_path, GEN, 32, device, edit=sharp, max_seq=256)
    kw.setdefault("max_seq_len", 256)
    kw.setdefault("dtype", torch.float32)
    return net, LocalEngine.create(net.path, device=torch.device(device), **kw)


def greedy(net, prompt, n):
    return oracle.greedy(prompt, n, net.W, GEN)


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation(tmp_path, device):
    net, eng = engine_for(tmp_path, device)
    prompt = toks(45, 272, 33)
    want = greedy(net, prompt, 40)
    out = eng.generate(prompt, max_new_tokens=40, stop_on_eos=False)
    assert out["token_ids"] == want
    # again on the same engine, and a shorter prompt after a longer one
    assert eng.generate(prompt, max_new_tokens=40,
                        stop_on_eos=False)["token_ids"] == want
    assert eng.generate(prompt[:3], max_new_tokens=12, stop_on_eos=False)[
        "token_ids"] == greedy(net, prompt[:3], 12)
    rows = [c["new_token_ids"] for c in eng.generate_stream(
        prompt, max_new_tokens=20, stop_on_eos=False, chunk=6)]
    assert sum(rows, []) == want[:20]
    # speculation asks for a cache that can go back: plain decoding instead
    assert eng.generate(prompt, max_new_tokens=20, stop_on_eos=False,
                        speculative=True)["token_ids"] == want[:20]


@pytest.mark.parametrize("device", DEVICES)
def test_prefill_in_slices(tmp_path, device, monkeypatch):
    net, eng = engine_for(tmp_path, device)
    monkeypatch.setattr(type(eng), "PREFILL_CHUNK", 32)
    prompt = toks(101, 272, 34)
    assert eng.generate(prompt, max_new_tokens=10, stop_on_eos=False)[
        "token_ids"] == greedy(net, prompt, 10)


@pytest.mark.parametrize("device", DEVICES)
def test_continuing_a_conversation(tmp_path, device):
    """A prefix is reused only where the state stands exactly behind it."""
    net, eng = engine_for(tmp_path, device)
    prompt = toks(30, 272, 35)
    first = eng.generate(prompt, max_new_tokens=9, stop_on_eos=False)
    longer = prompt + first["token_ids"][:-1] + toks(6, 272, 36)
    want = greedy(net, longer, 8)
    n = len(prompt) + 8
    out = eng.generate(longer, max_new_tokens=8, stop_on_eos=False, from_pos=n)
    assert out["token_ids"] == want and out["cached_prefix"] == n
    out = eng.generate(longer, max_new_tokens=8, stop_on_eos=False,
                       from_pos=20)
    assert out["token_ids"] == want and out["cached_prefix"] == 0
    with pytest.raises(ValueError):
        eng.prefill(longer[5:], from_pos=5)


@pytest.mark.parametrize("device", DEVICES)
def test_batch_generation_and_scoring(tmp_path, device):
    net, eng = engine_for(tmp_path, device, batch_size=3)
    prompts = [toks(n, 272, 37 + n) for n in (1, 40, 17)]
    rows = eng.generate_batch(prompts, max_new_tokens=12, stop_on_eos=False)
    for p, row in zip(prompts, rows):
        assert row["token_ids"] == greedy(net, p, 12)
    ids = prompts[1]
    ll = eng.loglikelihood(ids[:10], ids[10:])
    lp = torch.log_softmax(net.want(ids), -1)
    want = sum(float(lp[i - 1, ids[i]]) for i in range(10, len(ids)))
    assert abs(ll["logprob"] - want) < 1e-2


@pytest.mark.parametrize("device", DEVICES)
def test_sessions(tmp_path, device):
    """Continuous batching: prompts in portions beside decoding sessions,
    sessions that join, end and leave their blocks and slots to others."""
    from fei_amd.engine.sessions import PagedSessionManager, StepSessionManager
    net, eng = engine_for(tmp_path, device)
    mgr = PagedSessionManager(eng, num_blocks=6, max_sessions=3,
                              prefill_budget=16)
    assert isinstance(mgr, StepSessionManager)
    mgr.eos = -1                       # run to the length asked for
    prompts = [toks(n, 272, 40 + n) for n in (50, 3, 90, 20, 61)]
    want = [greedy(net, p, 15) for p in prompts]
    assert serve_sessions(mgr, prompts, 15) == want
    assert mgr.pool.free_blocks() == 6 and mgr.pool.free_slots() == 3


def test_end_of_the_positions(tmp_path):
    """Generation stops at the last position there is."""
    from fei_amd.engine.sessions import PagedSessionManager
    net, eng = engine_for(tmp_path, "cpu")
    prompt = toks(255, 272, 41)          # its end is kept, to leave room for 8
    out = eng.generate(prompt, max_new_tokens=8, stop_on_eos=False)
    assert out["token_ids"] == greedy(net, prompt[-247:], 8)
    mgr = PagedSessionManager(eng, max_sessions=2)
    mgr.eos = -1
    sid = mgr.open(toks(252, 272, 42), max_new_tokens=50)
    mgr.run()
    res = mgr.result(sid)
    assert res["done"] and len(res["token_ids"]) == 5
    with pytest.raises(ValueError):
        mgr.open(toks(256, 272, 43))
    with pytest.raises(ValueError):
        engine_for(tmp_path, "cpu", max_seq_len=257)


def test_served_over_http(tmp_path):
    from fastapi.testclient import TestClient

    from fei_amd.serve.api import create_app
    net, eng = engine_for(tmp_path, "cpu")
    client = TestClient(create_app(engine=eng, session_blocks=8))
    ids = eng.tokenizer.encode("hello")
    want = greedy(net, ids, 6)
    r = client.post("/v1/completions", json={
        "prompt": "hello", "max_tokens": 6, "stop_on_eos": False}).json()
    assert r["choices"][0]["text"] == eng.tokenizer.decode(want)
    sid = client.post("/v1/sessions", json={"prompt": "hello",
                                            "max_tokens": 6}).json()["session_id"]
    client.post("/v1/sessions/step?n=10")
    assert client.get(f"/v1/sessions/{sid}").json()["token_ids"][:3] == want[:3]
    client.delete(f"/v1/sessions/{sid}")


def test_unavailable_options_say_so():
    from fei_amd.engine.engine import LocalEngine
    from fei_amd.parallel.pg import ParallelContext
    spec = get_spec("bokenex-tiny")
    with pytest.raises(ValueError):
        LocalEngine(spec, device=torch.device("cpu"), weight_quant="fp8")
    with pytest.raises(ValueError):
        BokenexModel(spec, torch.device("cpu"),
                     tp=ParallelContext(rank=0, world_size=2))
    eng = LocalEngine(spec, device=torch.device("cpu"), max_seq_len=64)
    with pytest.raises(ValueError):
        eng.decode_speculative(4, [1, 2])


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("batch", [1, 3, 4])
def test_graph_replay_matches_eager(tmp_path, dtype, batch):
    """Captured decode steps against eager ones, with other work and
    synchronizations between the replays."""
    _, ge = engine_for(tmp_path, "cuda", dtype=dtype, batch_size=batch)
    _, ee = engine_for(tmp_path, "cuda", dtype=dtype, batch_size=batch,
                       use_hip_graph=False)
    prompt = toks(45, 272, 33)
    for eng in (ge, ee):
        eng.prefill(prompt)
    assert ge._graph is not None and ee._graph is None
    for _ in range(8):
        ge._graph.replay()
        torch.cuda.synchronize()
        ee._decode_step()
        torch.cuda.synchronize()
        a, b = ge._decode_logits(), ee._decode_logits()   # same position twice
        assert torch.equal(ge.token, ee.token)
        assert torch.equal(ge.pos, ee.pos)
        assert err(a, b.double().cpu()) < 1e-6
        for s, t in zip(ge.runner.cache.states, ee.runner.cache.states):
            assert torch.equal(s[:batch], t[:batch])


@pytest.mark.gpu
@pytest.mark.parametrize("batch", [1, 2, 8, 16])
def test_graph_replay_at_real_sizes(batch):
    """Skinny, tile and library products of a real layer, replayed with eager
    steps of another engine in between."""
    from dataclasses import replace

    from fei_amd.engine.engine import LocalEngine
    spec = get_spec("bokenex-1b")
    spec = replace(spec, name="two-layers", vocab_size=4096,
                   layers=spec.layers[:2])
    kw = dict(device=torch.device("cuda"), batch_size=batch, max_seq_len=1024,
              tokenizer=None)
    ge, ee = LocalEngine(spec, **kw), LocalEngine(spec, use_hip_graph=False,
                                                  **kw)
    prompt = toks(300, 4096, 45)
    for eng in (ge, ee):
        eng.prefill(prompt)
    for _ in range(6):
        ge._graph.replay()
        torch.cuda.synchronize()
        ee._decode_step()
        torch.cuda.synchronize()
        assert torch.equal(ge.token, ee.token)
        for a, b in zip(ge.runner.cache.rows, ee.runner.cache.rows):
            assert torch.equal(a[:64], b[:64])
    assert err(ge._decode_logits(), ee._decode_logits().double().cpu()) < 1e-6


# -- command line -----------------------------------------------------------------------

@pytest.mark.parametrize("device", DEVICES)
def test_trace_replay(tmp_path, device):
    net = Net(tmp_path / "m", make_cfg(
        [(att(6, 2, 24, 16, 30, 3), moe(4, 1, 40)), (att(), None)], width=64,
        vocab=96, positions=150), 44, device, max_seq=150)
    out = tmp_path / "out"
    out.mkdir()
    a, b = toks(90, 96, 1), toks(40, 96, 2)
    steps = [
        {"step": 0, "entries": [{"id": "x", "tokens": a[:70], "want": [69]}],
         "end": []},
        {"step": 1, "entries": [{"id": "y", "tokens": b[:39], "want": []},
                                {"id": "x", "tokens": a[70:71], "want": []}],
         "end": []},
        {"step": 2, "entries": [{"id": "x", "tokens": a[71:], "want": [0, 18]},
                                {"id": "y", "tokens": b[39:], "want": [0]}],
         "end": ["x", "y"]},
        {"step": 3, "entries": [{"id": "x", "tokens": b, "want": [39]}],
         "end": ["x"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    p = subprocess.run(
        [sys.executable, os.path.join(root, "bin", "trace_run"), "--model",
         net.path, "--dtype", "float32", "--out", str(out), "--max-tokens",
         "192", "--device", device],
        input="".join(json.dumps(s) + "\n" for s in steps),
        capture_output=True, text=True, timeout=100)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [ln for ln in p.stdout.splitlines() if ln.startswith("done")] == \
        [f"done {i}" for i in range(4)]
    wa, wb = net.want(a), net.want(b)
    want = {0: wa[[69]], 2: torch.stack([wa[71], wa[89], wb[39]]), 3: wb[[39]]}
    assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "3.f32"]
    for step, w in want.items():
        got = torch.from_numpy(np.fromfile(out / f"{step}.f32", dtype="<f4"))
        assert err(got.view(-1, 96), w) < F32_TOL


def test_listed_by_the_command_line(capsys):
    from fei_amd.ui.cli import main
    assert main(["models"]) == 0
    assert "bokenex-8b" in capsys.readouterr().out
