"""Plain, slow implementation of the Bokenex decoder, one function per
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


def rms_norm(x, g, eps):
    """x over its root mean square along the last dimension, times g (a
    number, or one per coordinate)."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * g


def embed(tokens, W):
    ids = torch.as_tensor(tokens, dtype=torch.long)
    return W["embed"][ids] + W["pos"][torch.arange(len(ids))]


def short_conv(u, w):
    """y_t = sum_j w[:, j] u_(t - taps + 1 + j) for u [T, channels]; nothing
    before t = 0."""
    taps = w.shape[1]
    y = torch.zeros_like(u)
    for t in range(u.shape[0]):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] += w[:, j] * u[s]
    return y


def distance_bias(d, r1, r2):
    """Taken off the score of a key d positions back."""
    return r1 * torch.log(1.0 + r2 * d)


def visible_keys(i, window):
    """Key positions that query position i sees."""
    return range(0 if window is None else max(0, i - window + 1), i + 1)


def key_weights(i, q, k, keys, scale, r1, r2, pb):
    """Weights of ``keys`` for the query q of position i; k [T, dim]."""
    d = i - torch.arange(keys.start, keys.stop, dtype=real)
    bias = distance_bias(d, r1, r2)
    return torch.sigmoid(k[keys.start:keys.stop] @ q * scale - bias + pb)


def attention(h, W, p, m, eps):
    """h [T, width], positions 0 .. T-1. m: sizes and constants."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    d, e = m["dim"], m["vdim"]
    q, k, v = (short_conv(h @ W[p + n].T, W[p + n + ".conv"]) for n in "qkv")
    q = rms_norm(q.view(T, H, d), W[p + "q.norm"], eps)
    k = rms_norm(k.view(T, G, d), W[p + "k.norm"], eps)
    v = v.view(T, G, e)
    window = (m.get("mask") or {}).get("size")
    out = torch.zeros(T, H, e, dtype=real)
    for i in range(T):
        keys = visible_keys(i, window)
        for hd in range(H):
            g = hd // (H // G)
            w = key_weights(i, q[i, hd], k[:, g], keys, m["scale"],
                            float(W[p + "r1"][hd]), float(W[p + "r2"][hd]),
                            float(W[p + "pb"][hd]))
            out[i, hd] = w @ v[keys.start:keys.stop, g]
    return out.view(T, H * e) @ W[p + "o"].T


def square_relu(z):
    return torch.clamp(z, min=0.0) ** 2


def two_layer(h, W, p):
    return square_relu(h @ W[p + "up"].T) @ W[p + "down"].T


def route(z, top, scale):
    """Router logits [experts] of one token -> [(expert, weight)]."""
    s = torch.sigmoid(z)
    best = sorted(range(len(s)), key=lambda e: -float(s[e]))[:top]
    total = sum(float(s[e]) for e in best) + 1e-20
    return [(e, float(s[e]) / total * scale) for e in best]


def experts(h, W, p, mlp):
    r = mlp["router"]
    z = h @ W[p + "router"].T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in route(z[t], r["top"], r["scale"]):
            out[t] += w * two_layer(h[t], W, f"{p}e{e}.")
    return out


def feed_forward(h, W, p, mlp):
    if mlp["kind"] == "moe":
        return experts(h, W, p, mlp)
    return two_layer(h, W, p)


def layer(x, W, i, cfg):
    L, p, eps = cfg["layers"][i], f"l{i}.", cfg["norm"]["eps"]
    h = rms_norm(x, W[p + "norm1"], eps)
    y = attention(h, W, p + "mix.", L["mixer"], eps)
    if L.get("mlp"):
        y = y + feed_forward(h, W, p + "mlp.", L["mlp"])
    return x + cfg["residual_mult"] * y


def forward(tokens, W, cfg, keep=None):
    """tokens -> logits [T, vocab]. ``keep``: a list that gets the residual
    after every layer."""
    x = embed(tokens, W)
    for i in range(len(cfg["layers"])):
        x = layer(x, W, i, cfg)
        if keep is not None:
            keep.append(x)
    return rms_norm(x, W["final.norm"], cfg["norm"]["eps"]) @ W["head"].T


def greedy(tokens, n, W, cfg):
    """n greedily chosen tokens after ``tokens``, whole context each time."""
    ids = list(tokens)
    for _ in range(n):
        ids.append(int(forward(ids, W, cfg)[-1].argmax()))
    return ids[len(tokens):]


# -- random models -----------------------------------------------------------

def tensor_shapes(cfg):
    """name -> shape of every tensor of a model with this configuration."""
    C = cfg["width"]
    out = {"embed": (cfg["vocab"], C), "pos": (cfg["max_positions"], C),
           "final.norm": (), "head": (cfg["vocab"], C)}
    for i, L in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", L["mixer"], L.get("mlp")
        H, G = m["heads"], m["kv_heads"]
        out[p + "norm1"] = ()
        for n, rows in (("q", H * m["dim"]), ("k", G * m["dim"]),
                        ("v", G * m["vdim"])):
            out[p + "mix." + n] = (rows, C)
            out[p + "mix." + n + ".conv"] = (rows, m["conv"])
        for n, size in (("q.norm", m["dim"]), ("k.norm", m["dim"]),
                        ("r1", H), ("r2", H), ("pb", H)):
            out[p + "mix." + n] = (size,)
        out[p + "mix.o"] = (C, H * m["vdim"])
        if not f:
            continue
        if f["kind"] == "dense":
            names, ff = [p + "mlp."], f["ff"]
        else:
            E, ff = f["router"]["experts"], f["expert"]["ff"]
            names = [f"{p}mlp.e{e}." for e in range(E)]
            out[p + "mlp.router"] = (E, C)
        for n in names:
            out[n + "up"] = (ff, C)
            out[n + "down"] = (C, ff)
    return out


def random_weights(cfg, seed):
    """bfloat16-valued float64 weights: gains around 1, distance biases of
    unlike strength, key weights around a tenth."""
    g = torch.Generator().manual_seed(seed)
    W = {}
    for name, shape in tensor_shapes(cfg).items():
        t = torch.randn(shape, generator=g)
        if name.endswith(("norm", "norm1")):
            t = 1.0 + 0.3 * t
        elif name.endswith(".r1"):
            t = t.abs()
        elif name.endswith(".r2"):
            t = 0.05 + 0.3 * t.abs()
        elif name.endswith(".pb"):
            t = -2.0 + 0.5 * t
        elif name.endswith(".conv"):
            t = t / math.sqrt(shape[-1])
        elif name.endswith("router"):
            t = t * (3.0 / math.sqrt(shape[-1]))   # choices far from a tie
        elif name in ("embed", "pos"):
            t = 0.7 * t
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
