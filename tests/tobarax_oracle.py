"""Plain, slow implementation of the Tobarax decoder, one function per
mechanism, written from its equations. It shares no code with fei_amd: the
tests compare the framework against it.

Everything runs in the dtype of ``real`` (float64 by default), one sequence
at a time, with Python loops over positions where that keeps an equation
readable.
"""

import json
import math
import os

import torch

real = torch.float64


def rms(x, eps):
    """x over its root mean square along the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return rms(x, eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def rotate_interleaved(x, positions, base):
    """x [T, ..., R]: each pair (2i, 2i+1) is turned by p * base^(-2i/R)."""
    R = x.shape[-1]
    out = x.clone()
    for i in range(R // 2):
        ang = positions.to(real) * (base ** (-2.0 * i / R))
        shape = [-1] + [1] * (x.dim() - 2)
        c, s = torch.cos(ang).view(shape), torch.sin(ang).view(shape)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def visible_keys(i, window):
    """Key positions that query position i sees."""
    lo = 0 if window is None else max(0, i - window + 1)
    return lo, i + 1


def latent_attention(h, W, p, m, eps):
    """h [T, C], positions 0..T-1. m: sizes and constants of the mixer."""
    T = h.shape[0]
    H, d, r, vd, kr = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(T)
    q = (h @ W[p + "q"].T).view(T, H, d + r)
    qn, qr = q[..., :d], q[..., d:]
    ckr = h @ W[p + "dkv"].T
    c = rms_norm(ckr[:, :kr], W[p + "dkv.norm"], eps)
    kr_ = ckr[:, kr:]
    if r:
        qr = rotate_interleaved(qr, pos, m["rot"]["base"])
        kr_ = rotate_interleaved(kr_, pos, m["rot"]["base"])
    k = (c @ W[p + "uk"].T).view(T, H, d)
    v = (c @ W[p + "uv"].T).view(T, H, vd)
    window = (m.get("mask") or {}).get("size")
    out = torch.zeros(T, H, vd, dtype=real)
    for i in range(T):
        lo, hi = visible_keys(i, window)
        for hd in range(H):
            s = (k[lo:hi, hd] @ qn[i, hd] + kr_[lo:hi] @ qr[i, hd]) * m["scale"]
            w = torch.softmax(s, 0)
            out[i, hd] = w @ v[lo:hi, hd]
    out = out.view(T, H * vd) * torch.sigmoid(h @ W[p + "g"].T)
    return out @ W[p + "o"].T


def gla_recurrence(q, k, v, alpha, S0=None):
    """q, k, alpha [T, H, d], v [T, H, e] -> o [T, H, e], last state."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=real) if S0 is None else S0.clone()
    o = torch.zeros(T, H, v.shape[-1], dtype=real)
    for t in range(T):
        S = alpha[t].unsqueeze(-1) * S + k[t].unsqueeze(-1) * v[t].unsqueeze(1)
        o[t] = (q[t].unsqueeze(-1) * S).sum(1)
    return o, S


def gla(h, W, p, m, eps):
    T = h.shape[0]
    H, d, e = m["heads"], m["dim"], m["vdim"]
    q = (h @ W[p + "q"].T).view(T, H, d) * d ** -0.5
    k = (h @ W[p + "k"].T).view(T, H, d)
    v = (h @ W[p + "v"].T).view(T, H, e)
    z = (h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "a2.b"]
    alpha = (torch.sigmoid(z) ** (1.0 / m["tau"])).view(T, H, d)
    o, _ = gla_recurrence(q, k, v, alpha)
    o = rms_norm(o, W[p + "norm"], eps).reshape(T, H * e)
    return (o * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


def feed_forward(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


MIXERS = {"latent_attention": latent_attention, "gla": gla}


def layer(x, W, i, cfg, eps):
    L = cfg["layers"][i]
    p = f"l{i}."
    y = MIXERS[L["type"]](rms_norm(x, W[p + "norm1"], eps), W, p + "mix.",
                          L["mixer"], eps)
    if L.get("mlp") is not None:
        y = y + feed_forward(rms_norm(x, W[p + "norm2"], eps), W, p + "mlp.")
    return x + y


def layer_runs(cfg):
    """[(layer, pass or None, first of its pass)] in the order they run."""
    loop = cfg.get("loop")
    n = len(cfg["layers"])
    if not loop:
        return [(i, None, False) for i in range(n)]
    a, b, times = loop["start"], loop["stop"], loop["times"]
    runs = [(i, None, False) for i in range(a)]
    for t in range(times):
        runs += [(i, t, i == a) for i in range(a, b)]
    return runs + [(i, None, False) for i in range(b, n)]


def head(x, W, cfg, eps):
    y = (rms_norm(x, W["final.norm"], eps) @ W["head"].T) * cfg["logit_scale"]
    cap = cfg.get("logit_softcap")
    return cap * torch.tanh(y / cap) if cap else y


def forward(tokens, W, cfg, keep=None):
    """tokens -> logits [T, vocab]. ``keep``: a list that gets the residual
    after every layer run."""
    eps = cfg["norm"]["eps"]
    x0 = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    x = x0
    for i, t, first in layer_runs(cfg):
        if first:
            x = torch.cat([x, x0], -1) @ W["loop.in"].T + W["loop.step"][t]
        x = layer(x, W, i, cfg, eps)
        if keep is not None:
            keep.append(x)
    return head(x, W, cfg, eps)


def greedy(tokens, n, W, cfg):
    """n greedily chosen tokens after ``tokens``, whole context each time."""
    ids = list(tokens)
    for _ in range(n):
        ids.append(int(forward(ids, W, cfg)[-1].argmax()))
    return ids[len(tokens):]


# -- random models -----------------------------------------------------------

def tensor_shapes(cfg, gate_rank=8):
    """name -> shape of every tensor of a model with this configuration."""
    C = cfg["width"]
    out = {"embed": (cfg["vocab"], C), "head": (cfg["vocab"], C),
           "final.norm": (C,)}
    if cfg.get("loop"):
        out["loop.in"] = (C, 2 * C)
        out["loop.step"] = (cfg["loop"]["times"], C)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        H = m["heads"]
        out[p + "norm1"] = (C,)
        if L["type"] == "latent_attention":
            out[p + "mix.q"] = (H * (m["dim"] + m["rot_dim"]), C)
            out[p + "mix.dkv"] = (m["kv_rank"] + m["rot_dim"], C)
            out[p + "mix.dkv.norm"] = (m["kv_rank"],)
            out[p + "mix.uk"] = (H * m["dim"], m["kv_rank"])
            out[p + "mix.uv"] = (H * m["vdim"], m["kv_rank"])
        else:
            out[p + "mix.q"] = (H * m["dim"], C)
            out[p + "mix.k"] = (H * m["dim"], C)
            out[p + "mix.v"] = (H * m["vdim"], C)
            out[p + "mix.norm"] = (m["vdim"],)
            out[p + "mix.a1"] = (gate_rank, C)
            out[p + "mix.a2"] = (H * m["dim"], gate_rank)
            out[p + "mix.a2.b"] = (H * m["dim"],)
        out[p + "mix.g"] = (H * m["vdim"], C)
        out[p + "mix.o"] = (C, H * m["vdim"])
        if L.get("mlp") is not None:
            out[p + "norm2"] = (C,)
            ff = L["mlp"]["ff"]
            out[p + "mlp.gate"] = (ff, C)
            out[p + "mlp.up"] = (ff, C)
            out[p + "mlp.down"] = (C, ff)
    return out


def random_weights(cfg, seed, gate_rank=8):
    """bfloat16-valued float64 weights; norms around 1, biases that give
    decays across (0, 1)."""
    g = torch.Generator().manual_seed(seed)
    W = {}
    for name, shape in tensor_shapes(cfg, gate_rank).items():
        t = torch.randn(*shape, generator=g)
        if name.endswith("norm") or name.endswith("norm1") or name.endswith("norm2"):
            t = 1.0 + 0.3 * t
        elif name.endswith("a2.b"):
            t = 1.0 + 2.0 * t
        elif name == "embed":
            t = 0.7 * t
        elif name == "loop.step":
            t = 0.3 * t
        else:
            t = t * (1.3 / math.sqrt(shape[-1]))
        W[name] = t.bfloat16().to(real)
    return W


def save_model(path, cfg, W):
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    save_file({k: v.bfloat16().contiguous() for k, v in W.items()},
              os.path.join(path, "model.safetensors"))
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
