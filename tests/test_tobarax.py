"""Tobarax against a plain implementation (tests/tobarax_oracle.py): every
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

import step_helpers
import tobarax_oracle as oracle
from fei_amd import ops
from fei_amd.engine.config import MODEL_SPECS, TobaraxSpec, get_spec
from fei_amd.engine.kv_cache import HybridCache
from fei_amd.engine.step import StepEntry
from fei_amd.models.tobarax import TobaraxModel
from step_helpers import (DEVICES, F32_TOL, err, run, run_mixed,
                          serve_sessions, toks)


def att(heads=3, dim=20, rot=6, vdim=28, kr=44, window=37, scale=None,
        base=9000.0):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim,
         "kv_rank": kr, "scale": scale or (dim + rot) ** -0.5,
         "rot": {"base": base, "dims": rot}}
    if window:
        m["mask"] = {"size": window}
    return m


def lin(heads=2, dim=12, vdim=20, tau=5.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}


def make_cfg(layers, width=52, vocab=101, loop=None, cap=9.0, scale=0.7):
    """layers: (mixer dict, ff or None) each; the mixer's keys tell its kind."""
    out = [{"type": "gla" if "tau" in m else "latent_attention", "mixer": m,
            "mlp": {"kind": "dense", "ff": ff} if ff else None}
           for m, ff in layers]
    cfg = {"architecture": "Tobarax", "layers": out, "logit_scale": scale,
           "logit_softcap": cap, "norm": {"eps": 3e-5}, "vocab": vocab,
           "width": width}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


CONFIGS = {
    # no size a multiple of 8, unlike layers, a layer without feed-forward, a
    # loop that starts after the first layer
    "odd": make_cfg([(att(), 36), (lin(), None), (att(2, 9, 10, 14, 33, 70,
                                                      base=400.0), 50),
                     (lin(3, 17, 11, 1.5), 21)], loop=(1, 3, 3)),
    # multiples of 8 (vector paths), more than 16 heads, a loop of one pass
    "even": make_cfg([(lin(2, 40, 72, 16.0), 64),
                      (att(18, 24, 8, 40, 72, 64), 96)], width=64, vocab=96,
                     loop=(0, 2, 1), cap=None, scale=1.0),
    # attention without a window, one head, no loop
    "full": make_cfg([(att(1, 40, 12, 56, 128, None), 40),
                      (lin(1, 64, 128, 8.0), 40)], width=48, vocab=77),
}


def Net(tmp, cfg, seed=0, device="cpu", dtype=torch.float32, edit=None,
        max_seq=512, gate_rank=5):
    return step_helpers.Net(tmp, oracle, cfg, seed, device, dtype, edit,
                            max_seq, gate_rank=gate_rank)


# -- mechanisms alone ------------------------------------------------------------

@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_every_layer_run(tmp_path, name, device):
    """The residual after each layer run: mixers, feed-forward, both norms,
    the entry of every pass."""
    net = Net(tmp_path, CONFIGS[name], 1, device)
    tokens = toks(70, net.cfg["vocab"], 2)
    keep, got = [], []
    oracle.forward(tokens, net.W, net.cfg, keep)
    r = net.runner()
    batch = r.build([StepEntry(r.admit(), tokens, [0])])
    with torch.no_grad():
        net.model.forward(batch, r.cache, lambda i, x: got.append(x.clone()))
    assert len(got) == len(keep) == len(get_spec(net.path).runs)
    for a, b in zip(got, keep):
        assert err(a, b) < F32_TOL


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("mixer", ["att", "gla"])
def test_mixer_alone(tmp_path, mixer, device):
    cfg = make_cfg([(att() if mixer == "att" else lin(), None)], cap=None)
    net = Net(tmp_path, cfg, 3, device)
    tokens = toks(150, cfg["vocab"], 4)
    r = net.runner()
    assert err(run(r, r.admit(), tokens, [150]), net.want(tokens)) < F32_TOL
    assert err(run(r, r.admit(), tokens, [1]), net.want(tokens)) < F32_TOL


def test_rotation_pairs_neighbours():
    x = torch.randn(9, 2, 10, dtype=torch.float64)
    pos = torch.arange(9) * 50
    table = ops.ref.rope_table_exact(500, 10, 700.0)
    got = ops.ref.apply_rope_interleaved(x, pos, table)
    want = oracle.rotate_interleaved(x, pos, 700.0)
    assert err(got.flatten(1), want.flatten(1)) < 1e-6


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("tau,bias", [(0.5, -25.0), (1.0, -4.0), (16.0, 6.0),
                                      (64.0, 14.0)])
def test_decay_from_forgetting_to_keeping(tmp_path, device, tau, bias):
    """Decays of e^-50 a token to 1 - 1e-8: nothing overflows, nothing is
    lost, in chunks and token by token. (With almost everything forgotten o is
    q.k times v, and the head norm magnifies the rounding of a small q.k.)"""
    tol = 5e-4 if bias < 0 else F32_TOL
    def edit(W):
        W["l0.mix.a2.b"] += bias
    cfg = make_cfg([(lin(2, 24, 20, tau), None)], cap=None)
    net = Net(tmp_path, cfg, 5, device, edit=edit)
    tokens = toks(150, cfg["vocab"], 6)
    r = net.runner()
    want = net.want(tokens)
    assert err(run(r, r.admit(), tokens, [150]), want) < tol
    assert err(run(r, r.admit(), tokens, [97, 1, 2]), want) < tol


@pytest.mark.parametrize("device", DEVICES)
def test_state_remembers_one_token(tmp_path, device):
    """Nearly no decay: an early token still shows hundreds of tokens later,
    across chunks, portions and decoding."""
    def edit(W):
        W["l0.mix.a2.b"] += 12.0
    cfg = make_cfg([(lin(1, 16, 16, 16.0), None)], cap=None)
    net = Net(tmp_path, cfg, 7, device, edit=edit)
    a = toks(300, cfg["vocab"], 8)
    b = [(a[0] + 1) % cfg["vocab"]] + a[1:]
    r = net.runner()
    la, lb = (run(r, r.admit(), t, [130, 64, 1, 1, 37])[-1] for t in (a, b))
    wa, wb = net.want(a)[-1], net.want(b)[-1]
    assert err((la - lb)[None], (wa - wb)[None]) < 1e-3
    assert float((wa - wb).norm() / wa.norm()) > 1e-3


@pytest.mark.parametrize("device", DEVICES)
def test_softcap_and_scale(device):
    y = torch.randn(5, 32)
    w = torch.randn(48, 32) * 3
    for scale, cap in ((0.3, 4.0), (2.0, None)):
        got = ops.logits_head(y.to(device), w.to(device), scale, cap)
        z = y.double() @ w.double().T * scale
        assert err(got, cap * torch.tanh(z / cap) if cap else z) < 1e-5


# -- prompts, decoding, portions ---------------------------------------------------

@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_prompt_decode_and_portions_agree(tmp_path, name, device):
    net = Net(tmp_path, CONFIGS[name], 9, device)
    tokens = toks(141, net.cfg["vocab"], 10)
    want = net.want(tokens)
    r = net.runner(slots=1)
    for sizes in ([141], [1], [2], [64], [63, 65], [2, 3, 5, 7, 1, 31],
                  [90, 1, 1, 2], [128, 1]):
        sid = r.admit()
        assert err(run(r, sid, tokens, sizes), want) < F32_TOL, sizes
        r.release(sid)


@pytest.mark.gpu
@pytest.mark.parametrize("name", list(CONFIGS))
def test_bfloat16(tmp_path, name):
    """The limits are 1.7 times what the reference ops give in bfloat16 on the
    CPU: 0.046 for the worst row and 0.018 overall, in the deepest model."""
    net = Net(tmp_path, CONFIGS[name], 9, "cuda", torch.bfloat16)
    tokens = toks(141, net.cfg["vocab"], 10)
    want = net.want(tokens)
    r = net.runner(slots=1)
    for sizes in ([141], [1], [2, 3, 61, 1]):
        sid = r.admit()
        got = run(r, sid, tokens, sizes)
        assert err(got, want) < 0.078, sizes
        assert err(got.flatten()[None], want.flatten()[None]) < 0.03, sizes
        r.release(sid)


@pytest.mark.parametrize("device", DEVICES)
def test_first_tokens(tmp_path, device):
    net = Net(tmp_path, CONFIGS["odd"], 11, device)
    r = net.runner()
    for n in (1, 2, 3):
        tokens = toks(n, net.cfg["vocab"], 20 + n)
        sid = r.admit()
        assert err(run(r, sid, tokens, [n]), net.want(tokens)) < F32_TOL
        r.release(sid)


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding(tmp_path, device):
    """Decoding past several windows, chunks and blocks."""
    net = Net(tmp_path, CONFIGS["odd"], 12, device)
    tokens = toks(330, net.cfg["vocab"], 13)
    r = net.runner()
    got = run(r, r.admit(), tokens, [30] + [1] * 300)
    assert err(got, net.want(tokens)) < F32_TOL


LARGE = {
    # the sizes of a real model's layers
    "usual": [att(16, 128, 64, 128, 512, 100), lin(4, 128, 256, 16.0)],
    # the largest sizes the kernels take
    "largest": [att(2, 192, 64, 256, 1024, 70), lin(2, 256, 512, 16.0)],
    # between the sizes that kernels are built for, vector paths
    "between": [att(5, 72, 24, 88, 136, 90), lin(3, 48, 104, 3.0)],
    # the same without them
    "ragged": [att(3, 67, 30, 85, 131, 90), lin(2, 45, 101, 3.0)],
}


@pytest.mark.gpu
@pytest.mark.parametrize("name", list(LARGE))
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_other_sizes(tmp_path, name, dtype):
    cfg = make_cfg([(m, None) for m in LARGE[name]], width=64, vocab=40)
    net = Net(tmp_path, cfg, 60, "cuda", dtype, gate_rank=16)
    tokens = toks(140, 40, 61)
    want = net.want(tokens)
    r = net.runner(slots=1)
    tol = F32_TOL if dtype == torch.float32 else 0.06
    for sizes in ([140], [131, 1], [5, 66, 1]):
        sid = r.admit()
        assert err(run(r, sid, tokens, sizes), want) < tol, sizes
        r.release(sid)


# -- single ops on the GPU ----------------------------------------------------------

@pytest.mark.gpu
@pytest.mark.parametrize("rows", [1, 2, 3, 4, 5, 8, 9, 33])
@pytest.mark.parametrize("width,n_mix,ff", [(1024, 96, 64), (2048, 144, 2048),
                                            (88, 30, 41), (52, 7, 0)])
def test_products(rows, width, n_mix, ff):
    """Every route of the skinny products against float64 on the same
    bfloat16 values: rows per wave, shared K, matrix tile, library."""
    g = torch.Generator().manual_seed(rows + width)
    bf = lambda *s: torch.randn(*s, generator=g).bfloat16()
    n1, n2 = bf(rows, width), bf(rows, width)
    w_in = bf(n_mix + 2 * ff, width) / width ** 0.5
    d = lambda t: t.double()
    cat = torch.zeros(rows, n_mix + ff, dtype=torch.bfloat16, device="cuda")
    proj = ops.mix_in(n1.cuda(), n2.cuda(), w_in.cuda(), n_mix, ff,
                      cat[:, n_mix:])
    assert err(proj, d(n1) @ d(w_in[:n_mix]).T) < 8e-3
    if ff:
        z = d(n2) @ d(w_in[n_mix:]).T
        act = z[:, :ff] * torch.sigmoid(z[:, :ff]) * z[:, ff:]
        assert err(cat[:, n_mix:], act) < 2e-2
    w = bf(n_mix + 50, width) / width ** 0.5
    x = torch.randn(rows, n_mix + 50, generator=g)
    y = ops.residual_linear(x.cuda(), n1.cuda(), w.cuda())
    assert err(y, d(x) + d(n1) @ d(w).T) < 1e-5
    b = torch.randn(n_mix + 50, generator=g)
    y = ops.linear_f32(n1.cuda(), w.cuda(), b.cuda())
    assert err(y, d(n1) @ d(w).T + d(b)) < 1e-5
    y = ops.logits_head(n1.cuda(), w.cuda(), 0.7, 2.0)
    assert err(y, 2.0 * torch.tanh(d(n1) @ d(w).T * 0.35)) < 1e-5


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("cols", [64, 77])
def test_row_ops(dtype, cols):
    g = torch.Generator().manual_seed(cols)
    x, y = (torch.randn(19, cols, generator=g) * 3 for _ in range(2))
    w1, w2 = torch.randn(cols, generator=g), torch.randn(cols, generator=g)
    tol = 1e-6 if dtype == torch.float32 else 4e-3
    a, b = ops.norm_pair(x.cuda(), w1.cuda(), w2.cuda(), 1e-3, dtype)
    want = oracle.rms(x.double(), 1e-3)
    assert a.dtype == dtype
    assert err(a, want * w1) < tol and err(b, want * w2) < tol
    assert ops.norm_pair(x.cuda(), w1.cuda(), None, 1e-3, dtype)[1] is None
    c = ops.cat_cast(x.cuda(), y.cuda(), dtype)
    assert torch.equal(c.cpu(), torch.cat([x, y], 1).to(dtype))


@pytest.mark.gpu
@pytest.mark.parametrize("batch", [3, 12])
@pytest.mark.parametrize("vocab", [4096, 1003])
def test_sampling_of_float32_logits(batch, vocab):
    """Differences below bfloat16's resolution decide."""
    g = torch.Generator().manual_seed(vocab)
    logits = torch.rand(batch, vocab, generator=g)
    best = torch.randint(0, vocab, (batch,), generator=g)
    logits[torch.arange(batch), best] = 1.0001
    logits[torch.arange(batch), (best + 1) % vocab] = 1.0
    token = torch.zeros(batch, dtype=torch.int32, device="cuda")
    step = torch.zeros(1, dtype=torch.int32, device="cuda")
    ws = torch.zeros(batch, 128, device="cuda")
    outs = torch.zeros(batch, 4, dtype=torch.int32, device="cuda")
    ops.sample(logits.cuda(), token, step, ws, out_tokens=outs)
    assert token.tolist() == best.tolist() == outs[:, 0].tolist()
    ops.sample(logits.cuda() * 4, token, step, ws, temperature=0.8, seed=11)
    noisy = logits * 5.0 + ops.ref.hash_gumbel(batch, vocab, 0, 11, 0)
    for i, t in enumerate(token.tolist()):
        assert float(noisy[i, t]) > float(noisy[i].max()) - 1e-3


# -- window edges -------------------------------------------------------------------

def every_key_counts(W):
    """Even weights, so that no key of a window is without any, and values
    that outweigh the residual."""
    W["l0.mix.q"] *= 0.5
    W["l0.mix.uv"] *= 8.0


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("window", [1, 2, 63, 64, 65, 100, 128])
def test_window_edge(tmp_path, window, device):
    """Changing the token just inside the window changes the output of one
    attention layer; just outside it changes nothing. In a prompt, in
    portions and in decoding, with queries around block borders."""
    cfg = make_cfg([(att(2, 16, 8, 16, 24, window), None)], width=32,
                   vocab=71, cap=None)
    net = Net(tmp_path, cfg, 14, device, edit=every_key_counts)
    a = toks(200, cfg["vocab"], 15)
    r = net.runner(slots=1)

    def logits(tokens, sizes):
        sid = r.admit()
        out = run(r, sid, tokens, sizes)
        r.release(sid)
        return out

    schedules = ([200], [70, 1, 1, 40, 2], [1])
    base = [logits(a, s) for s in schedules]
    want = net.want(a)
    for s, x in zip(schedules, base):
        assert err(x, want) < F32_TOL, s
    for q in (127, 128, 129, 191, 192, 199):
        for inside in (True, False):
            k = q - window + (1 if inside else 0)
            if k < 0 or k == q:
                continue
            # of some tokens at place k, the one that moves the output most
            moved, b, new = max(
                (((y - want[q]).norm() / want[q].norm()).item(), c, y)
                for c, y in ((c, net.want(c)[q]) for c in (
                    a[:k] + [(a[k] + d) % cfg["vocab"]] + a[k + 1:q + 1]
                    for d in (7, 19, 40, 66))))
            assert moved > 20 * F32_TOL if inside else moved < 1e-12
            for s in schedules:
                assert err(logits(b, s)[q][None], new[None]) < F32_TOL, (q, s)


@pytest.mark.parametrize("device", DEVICES)
def test_far_key_among_many(tmp_path, device):
    """One key far back that takes nearly all the weight, at block borders."""
    cfg = make_cfg([(att(1, 16, 0, 16, 24, None, scale=1.0), None)], cap=None)

    def edit(W):
        W["l0.mix.q"] *= 3.0
        W["l0.mix.uk"] *= 3.0
    net = Net(tmp_path, cfg, 16, device, edit=edit)
    r = net.runner(slots=1)
    for k in (0, 63, 64, 127, 128):
        tokens = toks(260, cfg["vocab"] - 1, 17)
        tokens[k] = cfg["vocab"] - 1          # a token seen once
        sid = r.admit()
        got = run(r, sid, tokens, [200, 1, 1, 30, 28])
        r.release(sid)
        assert err(got, net.want(tokens)) < 1e-4


# -- batches, blocks and slots ---------------------------------------------------------

@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", ["odd", "even"])
def test_mixed_batches(tmp_path, name, device):
    """Unequal requests in one batch, portions beside single tokens, requests
    that pause, end and make room for others."""
    net = Net(tmp_path, CONFIGS[name], 18, device)
    V = net.cfg["vocab"]
    reqs = {i: toks(n, V, 30 + i) for i, n in enumerate((150, 97, 64, 33, 120))}
    want = {i: net.want(t) for i, t in reqs.items()}
    r = net.runner(blocks=8, slots=3)
    got = run_mixed(r, reqs)
    for i in reqs:
        assert err(got[i], want[i]) < F32_TOL, i
    assert r.cache.free_blocks() == 8 and r.cache.free_slots() == 3


@pytest.mark.parametrize("device", DEVICES)
def test_wanted_rows_follow_the_entries(tmp_path, device):
    """Logits come in the order of the entries although single tokens are
    packed first."""
    net = Net(tmp_path, CONFIGS["even"], 19, device)
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


@pytest.mark.parametrize("device", DEVICES)
def test_blocks_and_slots_used_again(tmp_path, device):
    """Two sequences in a row on the same block and slot, in both orders."""
    net = Net(tmp_path, CONFIGS["odd"], 21, device)
    V = net.cfg["vocab"]
    r = net.runner(blocks=2, slots=1)
    for seed, sizes in ((1, [100]), (2, [1]), (3, [7, 64]), (4, [90, 1])):
        tokens = toks(100, V, seed)
        sid = r.admit()
        assert err(run(r, sid, tokens, sizes), net.want(tokens)) < F32_TOL
        with pytest.raises(MemoryError):
            r.admit()
        r.release(sid)


def test_cache_limits_and_fork():
    c = HybridCache([6, None], [None, (2, 3, 4)], num_blocks=3, num_slots=2,
                    block_size=4, dtype=torch.float32)
    a = c.new_sequence()
    c.ensure_capacity(a, 7)
    for i, blk in enumerate(c.table(a).blocks):
        c.rows[0].view(-1, 4, 6)[blk] = i + 1.0
    c.states[1][c.slot(a)] = 5.0
    with pytest.raises(MemoryError):
        c.fork(a)                              # one block left, two needed
    assert c.free_blocks() == 1 and c.free_slots() == 1
    c.release(a)
    a = c.new_sequence()
    c.ensure_capacity(a, 4)
    c.rows[0].view(-1, 4, 6)[c.table(a).blocks[0]] = 9.0
    c.states[1][c.slot(a)] = 7.0
    b = c.fork(a)
    assert c.table(b).blocks != c.table(a).blocks
    assert bool((c.rows[0].view(-1, 4, 6)[c.table(b).blocks[0]] == 9.0).all())
    assert bool((c.states[1][c.slot(b)] == 7.0).all())
    with pytest.raises(MemoryError):
        c.new_sequence()
    c.release(a)
    c.release(b)
    assert c.free_blocks() == 3 and c.free_slots() == 2


def test_step_refuses_bad_entries(tmp_path):
    net = Net(tmp_path, CONFIGS["full"], 22, max_seq=64)
    r = net.runner()
    s = r.admit()
    for entry in (StepEntry(s, []), StepEntry(s, [net.cfg["vocab"]]),
                  StepEntry(s, [1], [1]), StepEntry(s, [1] * 65)):
        with pytest.raises(ValueError):
            r.step([entry])
    with pytest.raises(ValueError):
        r.step([StepEntry(s, [1]), StepEntry(s, [2])])
    assert r.length[s] == 0


# -- configuration and weights ------------------------------------------------------

def test_config_round_trip(tmp_path):
    net = Net(tmp_path / "a", CONFIGS["odd"], 23)
    net.model.save_weights(str(tmp_path / "b"))
    spec = get_spec(str(tmp_path / "b"))
    assert spec.layers == net.model.spec.layers
    assert spec.loop == net.model.spec.loop
    again = TobaraxModel(spec, torch.device("cpu"), torch.float32,
                         weights=str(tmp_path / "b"))
    for k, v in net.model.state_dict_full().items():
        assert torch.equal(v, again.state_dict_full()[k]), k
        assert torch.equal(v.double(), net.W[k]), k


def test_unknown_config_is_refused(tmp_path):
    shapes = {f"l{i}.mix.a1": (5, 52) for i in range(4)}
    for path, value in ((("layers", 0, "mixer", "bias"), True),
                        (("layers", 0, "type"), "other"),
                        (("layers", 0, "mlp", "kind"), "other"),
                        (("layers", 0, "mixer", "rot", "dims"), 4),
                        (("extra",), 1), (("loop", "stop"), 9)):
        cfg = json.loads(json.dumps(CONFIGS["odd"]))
        d = cfg
        for k in path[:-1]:
            d = d[k]
        d[path[-1]] = value
        with pytest.raises(ValueError):
            TobaraxSpec.from_config(cfg, shapes)
    with pytest.raises(KeyError):
        get_spec(str(tmp_path))


def test_wrong_tensors_are_refused(tmp_path):
    from safetensors.torch import load_file, save_file
    net = Net(tmp_path, CONFIGS["full"], 24)
    f = os.path.join(net.path, "model.safetensors")
    full = load_file(f)
    missing = {k: v for k, v in full.items() if k != "l0.mix.g"}
    extra = dict(full, other=torch.zeros(1))
    shape = dict(full, head=torch.zeros(3, 48, dtype=torch.bfloat16))
    for bad in (missing, extra, shape):
        save_file(bad, f)
        with pytest.raises(ValueError):
            TobaraxModel(net.model.spec, torch.device("cpu"), torch.float32,
                         weights=net.path)


def test_registered_specs():
    for name, spec in MODEL_SPECS.items():
        if spec.arch == "tobarax":
            assert spec.params_bytes() > 0 and get_spec(name) is spec
    m = TobaraxModel(get_spec("tobarax-tiny"), torch.device("cpu"),
                     torch.float32, seed=3)
    assert m.param_bytes() == 4 * sum(
        t.numel() for t in m.state_dict_full().values())
    assert m.cache_bytes_per_token() == 4 * 64 * 2     # two attention runs


# -- generation ----------------------------------------------------------------------

GEN = make_cfg([(att(2, 16, 8, 24, 40, 30), 48), (lin(2, 16, 24, 4.0), 48)],
               width=64, vocab=272, loop=(0, 2, 2))


def sharp(W):
    """Logits far enough apart that rounding does not change the largest."""
    W["head"] *= 3.0


def engine_for(tmp_path, device, **kw):
    from fei_amd.engine.engine import LocalEngine
    net = Net(tmp_path, GEN, 25, device, edit=sharp)
    kw.setdefault("max_seq_len", 256)
    eng = LocalEngine.create(net.path, device=torch.device(device),
                             dtype=torch.float32, **kw)
    return net, eng


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation(tmp_path, device):
    net, eng = engine_for(tmp_path, device)
    prompt = toks(45, 272, 26)
    want = oracle.greedy(prompt, 40, net.W, GEN)
    out = eng.generate(prompt, max_new_tokens=40, stop_on_eos=False)
    assert out["token_ids"] == want
    # again on the same engine, and a shorter prompt after a longer one
    assert eng.generate(prompt, max_new_tokens=40,
                        stop_on_eos=False)["token_ids"] == want
    assert eng.generate(prompt[:3], max_new_tokens=12, stop_on_eos=False)[
        "token_ids"] == oracle.greedy(prompt[:3], 12, net.W, GEN)
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
    prompt = toks(101, 272, 27)
    assert eng.generate(prompt, max_new_tokens=10, stop_on_eos=False)[
        "token_ids"] == oracle.greedy(prompt, 10, net.W, GEN)


@pytest.mark.parametrize("device", DEVICES)
def test_continuing_a_conversation(tmp_path, device):
    """A prefix is reused only where the state stands exactly behind it."""
    net, eng = engine_for(tmp_path, device)
    prompt = toks(30, 272, 28)
    first = eng.generate(prompt, max_new_tokens=9, stop_on_eos=False)
    longer = prompt + first["token_ids"][:-1] + toks(6, 272, 29)
    want = oracle.greedy(longer, 8, net.W, GEN)
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
    prompts = [toks(n, 272, 31 + n) for n in (1, 40, 17)]
    rows = eng.generate_batch(prompts, max_new_tokens=12, stop_on_eos=False)
    for p, row in zip(prompts, rows):
        assert row["token_ids"] == oracle.greedy(p, 12, net.W, GEN)
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
    want = [oracle.greedy(p, 15, net.W, GEN) for p in prompts]
    assert serve_sessions(mgr, prompts, 15) == want
    assert mgr.pool.free_blocks() == 6 and mgr.pool.free_slots() == 3


def test_session_at_the_end_of_its_room(tmp_path):
    from fei_amd.engine.sessions import PagedSessionManager
    net, eng = engine_for(tmp_path, "cpu", max_seq_len=32)
    mgr = PagedSessionManager(eng, max_sessions=2)
    mgr.eos = -1
    sid = mgr.open(toks(28, 272, 50), max_new_tokens=50)
    mgr.run()
    res = mgr.result(sid)
    assert res["done"] and len(res["token_ids"]) == 5
    with pytest.raises(ValueError):
        mgr.open(toks(32, 272, 51))


def test_served_over_http(tmp_path):
    from fastapi.testclient import TestClient

    from fei_amd.serve.api import create_app
    net, eng = engine_for(tmp_path, "cpu")
    client = TestClient(create_app(engine=eng, session_blocks=8))
    ids = eng.tokenizer.encode("hello")
    want = oracle.greedy(ids, 6, net.W, GEN)
    r = client.post("/v1/completions", json={
        "prompt": "hello", "max_tokens": 6, "stop_on_eos": False}).json()
    assert r["choices"][0]["text"] == eng.tokenizer.decode(want)
    sid = client.post("/v1/sessions", json={"prompt": "hello",
                                            "max_tokens": 6}).json()["session_id"]
    client.post("/v1/sessions/step?n=10")
    assert client.get(f"/v1/sessions/{sid}").json()["token_ids"][:3] == want[:3]
    client.delete(f"/v1/sessions/{sid}")


def test_unavailable_options_say_so(tmp_path):
    from fei_amd.engine.engine import LocalEngine
    from fei_amd.parallel.pg import ParallelContext
    spec = get_spec("tobarax-tiny")
    with pytest.raises(ValueError):
        LocalEngine(spec, device=torch.device("cpu"), weight_quant="fp8")
    with pytest.raises(ValueError):
        TobaraxModel(spec, torch.device("cpu"),
                     tp=ParallelContext(rank=0, world_size=2))
    eng = LocalEngine(spec, device=torch.device("cpu"), max_seq_len=64)
    with pytest.raises(ValueError):
        eng.decode_speculative(4, [1, 2])


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("batch", [1, 3])
def test_graph_replay_matches_eager(tmp_path, dtype, batch):
    """Captured decode steps against eager ones, with other work and
    synchronizations between the replays."""
    from fei_amd.engine.engine import LocalEngine
    net = Net(tmp_path, GEN, 25, "cuda", edit=sharp)
    kw = dict(device=torch.device("cuda"), dtype=dtype, batch_size=batch,
              max_seq_len=256)
    ge = LocalEngine.create(net.path, **kw)
    ee = LocalEngine.create(net.path, use_hip_graph=False, **kw)
    prompt = toks(45, 272, 26)
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
            if s is not None:       # the extra step changed both alike
                assert torch.equal(s[:batch], t[:batch])


# -- the trace runner -------------------------------------------------------------------

@pytest.mark.parametrize("device", DEVICES)
def test_trace_replay(tmp_path, device):
    net = Net(tmp_path / "m", CONFIGS["even"], 26)
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
