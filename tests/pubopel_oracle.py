"""Plain float64 implementation of the Pubopel decoder, whole sequences only:
one function per mechanism, numpy, no code shared with the engine. Weights
are a dict of checkpoint names -> arrays, sizes and constants the config dict.

Notation: T tokens, C model width, H query heads, G key/value heads, D head
size, E experts.
"""
from __future__ import annotations

import numpy as np


def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def dyt(x, W, name):
    """Dynamic tanh: a squashing function in the place of a norm."""
    return np.tanh(W[name + ".alpha"].reshape(()) * x) * W[name] + W[name + ".b"]


def row_rms_norm(x, w, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * w


def input_convolution(h, w):
    """h plus a causal convolution of it, channel by channel; w [C, taps], the
    last tap meets the current token."""
    taps = w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, h.shape[1])), h])
    y = h.copy()
    for j in range(taps):
        y = y + w[:, j] * padded[j : j + h.shape[0]]
    return y


def visible_keys(T, mask):
    """bool [T, T]: query i (row) sees key j (column)."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    seen = j <= i
    if mask:
        seen &= (i - j < int(mask["size"])) | (j < int(mask.get("keep_first", 0)))
    return seen


def head_slope(h, H):
    return 2.0 ** (-8.0 * (h + 1) / H)


def head_attention(q, k, v, scale, temp, softcap, slope, sink, seen):
    """One head: q, k [T, D], v [T, Dv] -> [T, Dv]."""
    T = q.shape[0]
    s = (q @ k.T) * scale * temp
    if softcap:
        s = softcap * np.tanh(s / softcap)
    s = s - slope * (np.arange(T)[:, None] - np.arange(T)[None, :])
    s = np.where(seen, s, -np.inf)
    top = np.maximum(s.max(-1, keepdims=True), sink)
    p = np.exp(s - top)
    return (p @ v) / (p.sum(-1, keepdims=True) + np.exp(sink - top))


def attention(h, W, pre, m, eps):
    T = h.shape[0]
    H, G, D = int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    q, k = h @ W[pre + "q"].T, h @ W[pre + "k"].T
    v = k.reshape(T, G, D)
    q = row_rms_norm(q, W[pre + "q.norm"], eps).reshape(T, H, D)
    k = row_rms_norm(k, W[pre + "k.norm"], eps).reshape(T, G, D)
    seen = visible_keys(T, m.get("mask"))
    out = np.zeros((T, H, D))
    for hd in range(H):
        g = hd // (H // G)
        out[:, hd] = head_attention(
            q[:, hd], k[:, g], v[:, g], float(m["scale"]), float(W[pre + "temp"][hd]),
            float(m.get("softcap") or 0.0), head_slope(hd, H),
            float(W[pre + "sink"][hd]), seen)
    return out.reshape(T, H * D) @ W[pre + "o"].T


def gated_expert(h, W, pre):
    z = h @ W[pre + "gate"].T
    return (z * sigmoid(z) * (h @ W[pre + "up"].T)) @ W[pre + "down"].T


def routed_ff(h, W, pre, mlp):
    """A chosen expert sees the token times its own score."""
    top = int(mlp["router"]["top"])
    s = sigmoid(h @ W[pre + "router"].T)
    out = np.zeros((h.shape[0], W[pre + "e0.down"].shape[0]))
    for t in range(h.shape[0]):
        for e in np.argsort(-s[t], kind="stable")[:top]:
            out[t] += gated_expert(s[t, e] * h[t : t + 1], W, f"{pre}e{e}.")[0]
    if mlp.get("shared"):
        out += gated_expert(h, W, pre + "shared.")
    return out


def forward(cfg, W, tokens, layers_out=None):
    """Logits [T, vocab] of one whole sequence. layers_out (a list) receives
    the residual after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = W["embed"][np.asarray(tokens)]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        assert L["type"] == "attention"
        h = input_convolution(dyt(x, W, p + "norm1"), W[p + "canon1"])
        x = x + dyt(attention(h, W, p + "mix.", L["mixer"], eps), W, p + "norm1b")
        if L.get("mlp") is not None:
            h = input_convolution(dyt(x, W, p + "norm2"), W[p + "canon2"])
            x = x + dyt(routed_ff(h, W, p + "mlp.", L["mlp"]), W, p + "norm2b")
        if layers_out is not None:
            layers_out.append(x)
    return dyt(x, W, "final.norm") @ W["head"].T


def random_weights(cfg, seed):
    """{name: bfloat16 torch tensor} for a config."""
    import torch

    g = torch.Generator().manual_seed(seed)
    W = {}

    def mat(name, n_out, n_in, gain=1.0):
        W[name] = (torch.randn(n_out, n_in, generator=g) * gain * n_in ** -0.5).bfloat16()

    def vec(name, n, center, spread=0.2):
        W[name] = (center + spread * torch.randn(n, generator=g)).bfloat16()

    def norm(name, n, alpha):
        vec(name, n, 1.0)
        vec(name + ".b", n, 0.0)
        W[name + ".alpha"] = torch.tensor(alpha).bfloat16()

    width, vocab, taps = cfg["width"], cfg["vocab"], int(cfg["canon"]["taps"])
    W["embed"] = torch.randn(vocab, width, generator=g).bfloat16()
    mat("head", vocab, width, 2.0)
    norm("final.norm", width, 0.6)
    for i, L in enumerate(cfg["layers"]):
        p, m, q = f"l{i}.", L["mixer"], f"l{i}.mix."
        for n in (1, 2):
            if n == 2 and L.get("mlp") is None:
                continue
            norm(f"{p}norm{n}", width, 0.4 + 0.1 * n + 0.05 * i)
            norm(f"{p}norm{n}b", width, 0.9 - 0.1 * n)
            W[f"{p}canon{n}"] = (0.4 * torch.randn(width, taps, generator=g)).bfloat16()
        H, G, D = m["heads"], m["kv_heads"], m["dim"]
        mat(q + "q", H * D, width, 2.0)
        mat(q + "k", G * D, width, 2.0)
        vec(q + "q.norm", H * D, 1.2, 0.4)
        vec(q + "k.norm", G * D, 1.2, 0.4)
        vec(q + "temp", H, 1.1, 0.5)
        vec(q + "sink", H, 0.5, 1.0)
        mat(q + "o", width, H * D)
        mlp = L.get("mlp")
        if mlp is None:
            continue
        q = p + "mlp."
        names = [f"{q}e{e}." for e in range(mlp["router"]["experts"])]
        sizes = [mlp["expert"]["ff"]] * len(names)
        if mlp.get("shared"):
            names.append(q + "shared.")
            sizes.append(mlp["shared"]["ff"])
        for n, ff in zip(names, sizes):
            mat(n + "gate", ff, width, 3.0)
            mat(n + "up", ff, width, 3.0)
            mat(n + "down", width, ff)
        mat(q + "router", mlp["router"]["experts"], width, 3.0)
    return W


def as_float64(W):
    return {k: v.double().numpy() for k, v in W.items()}
