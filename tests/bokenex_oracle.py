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


def distance_bias(i, j, r1, r2):
    return r1 * math.log(1.0 + r2 * (i - j))


def visible_keys(i, window):
    """Key positions that query position i sees."""
    return range(0 if window is None else max(0, i - window + 1), i + 1)


def key_weights(i, q, k, keys, scale, r1, r2, pb):
    """Weights of ``keys`` for the query q of position i; k [T, dim]."""
    bias = torch.tensor([distance_bias(i, j, r1, r2) for j in keys],
                        dtype=real)
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
