"""Plain whole-sequence implementation of the Lipulorn decoder, one function
per mechanism, float64 numpy throughout, no cache, no state slots and no
batching. It exists to be compared with the engine and shares no code with it.

A model is (cfg, W): cfg the parsed config.json, W {tensor name: float64
array}. Every function takes whole-sequence arrays [n, ...].
"""
from __future__ import annotations

import numpy as np


def unit_rms(x, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    return unit_rms(x, eps) * w


def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return np.logaddexp(0.0, x)


# ---------------------------------------------------------------------------
# softmax attention: what a position sees
# ---------------------------------------------------------------------------
def window_mask(n, size):
    """[n, n] bool: the token itself and the size - 1 before it (size 0: all)."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    return (j <= i) & ((i - j < size) if size else True)


def chunk_mask(n, size):
    """[n, n] bool: earlier tokens of the position-aligned chunk (size 0: all)."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    return (j <= i) & ((i // size == j // size) if size else True)


def masked_softmax(scores, seen):
    s = np.where(seen, scores, -np.inf)
    e = np.exp(s - s.max(-1, keepdims=True))
    return e / e.sum(-1, keepdims=True)


def rotate_halves(x, pos, base):
    """x [n, ..., dims]: dimension i is paired with i + dims / 2."""
    dims = x.shape[-1]
    half = dims // 2
    f = np.array([base ** (-2.0 * i / dims) for i in range(half)])
    a = np.asarray(pos, dtype=np.float64).reshape((-1,) + (1,) * (x.ndim - 1)) * f
    u, v = x[..., :half], x[..., half:]
    return np.concatenate([u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a)], -1)


def chunked_attention(h, W, p, mx, eps):
    """Grouped heads, biased projections, unit-RMS queries and keys, chunks,
    one output gate per head."""
    n = h.shape[0]
    H, G, D, Dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = unit_rms((h @ W[p + "q"].T + W[p + "q.b"]).reshape(n, H, D), eps)
    k = unit_rms((h @ W[p + "k"].T + W[p + "k.b"]).reshape(n, G, D), eps)
    v = (h @ W[p + "v"].T + W[p + "v.b"]).reshape(n, G, Dv)
    seen = chunk_mask(n, mx["mask"]["size"])
    gate = sigmoid(h @ W[p + "g"].T)
    out = np.zeros((n, H, Dv))
    for hd in range(H):
        kv = hd // (H // G)
        a = masked_softmax(q[:, hd] @ k[:, kv].T * mx["scale"], seen)
        out[:, hd] = (a @ v[:, kv]) * gate[:, hd : hd + 1]
    return out.reshape(n, H * Dv) @ W[p + "o"].T


def latent_rows(h, W, p, mx, eps):
    """(latent [n, kv_rank], rotated key part [n, rot_dim]) of a layer that
    makes its own."""
    R = mx["kv_rank"]
    down = h @ W[p + "dkv"].T
    return (rms_norm(down[:, :R], W[p + "dkv.norm"], eps),
            rotate_halves(down[:, R:], np.arange(h.shape[0]), mx["rot"]["base"]))


def latent_attention(h, W, p, mx, eps, rows):
    """rows: what latent_rows gave, here or in the layer it is taken from."""
    n = h.shape[0]
    H, D, Dr, Dv = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"]
    c, k_rot = rows
    q = rms_norm(h @ W[p + "dq"].T, W[p + "dq.norm"], eps) @ W[p + "uq"].T
    q = q.reshape(n, H, D + Dr)
    q_rot = rotate_halves(q[..., D:], np.arange(n), mx["rot"]["base"])
    k = (c @ W[p + "uk"].T).reshape(n, H, D)
    v = (c @ W[p + "uv"].T).reshape(n, H, Dv)
    seen = window_mask(n, mx["mask"]["size"])
    out = np.zeros((n, H, Dv))
    for hd in range(H):
        s = (q[:, hd, :D] @ k[:, hd].T + q_rot[:, hd] @ k_rot.T) * mx["scale"]
        out[:, hd] = masked_softmax(s, seen) @ v[:, hd]
    return out.reshape(n, H * Dv) @ W[p + "o"].T


# ---------------------------------------------------------------------------
# gated delta rule with a decay per key channel
# ---------------------------------------------------------------------------
def short_conv_silu(x, w):
    """x [n, C], w [C, taps]: the last column weighs the current token."""
    n, taps = x.shape[0], w.shape[1]
    y = np.zeros_like(x)
    for t in range(n):
        for j in range(taps):
            src = t - (taps - 1) + j
            if src >= 0:
                y[t] += w[:, j] * x[src]
    return silu(y)


def unit_vectors(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def channel_decay(pre, a_log, dt_bias):
    """pre [n, H * D] -> decay factors [n, H, D]; a_log [H], dt_bias [H * D]."""
    H = a_log.shape[0]
    rate = softplus(pre + dt_bias).reshape(pre.shape[0], H, -1)
    return np.exp(-np.exp(a_log)[:, None] * rate)


def delta_recurrence(q, k, v, beta, g):
    """One head: q, k, g [n, D], v [n, Dv], beta [n]. Returns o [n, Dv]."""
    S = np.zeros((q.shape[1], v.shape[1]))
    o = np.zeros_like(v)
    for t in range(q.shape[0]):
        S = g[t][:, None] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + np.outer(k[t], u)
        o[t] = S.T @ q[t]
    return o


def delta_mixer(h, W, p, mx, eps):
    n = h.shape[0]
    H, G, D, Dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = short_conv_silu(h @ W[p + "q"].T, W[p + "q.conv"]).reshape(n, G, D)
    k = short_conv_silu(h @ W[p + "k"].T, W[p + "k.conv"]).reshape(n, G, D)
    v = short_conv_silu(h @ W[p + "v"].T, W[p + "v.conv"]).reshape(n, H, Dv)
    q = unit_vectors(q) * D ** -0.5
    k = unit_vectors(k)
    beta = sigmoid(h @ W[p + "b"].T)
    g = channel_decay(h @ W[p + "a1"].T @ W[p + "a2"].T, W[p + "A_log"], W[p + "dt_bias"])
    out = np.zeros((n, H, Dv))
    for hd in range(H):
        kv = hd // (H // G)
        out[:, hd] = delta_recurrence(q[:, kv], k[:, kv], v[:, hd], beta[:, hd], g[:, hd])
    out = rms_norm(out, W[p + "norm"], eps).reshape(n, H * Dv)
    return (out * sigmoid(h @ W[p + "g1"].T @ W[p + "g2"].T)) @ W[p + "o"].T


# ---------------------------------------------------------------------------
# feed-forward, streams, the model
# ---------------------------------------------------------------------------
def dense_feed_forward(h, W, p):
    a = silu(h @ W[p + "gate"].T + W[p + "gate.b"]) * (h @ W[p + "up"].T + W[p + "up.b"])
    return a @ W[p + "down"].T + W[p + "down.b"]


def read_streams(X, read):
    """X [n, S, width]."""
    return sum(read[s] * X[:, s] for s in range(X.shape[1]))


def write_streams(X, y, mix, write):
    """mix [from, to]; every new stream is made of the old ones."""
    S = X.shape[1]
    return np.stack([sum(mix[s, t] * X[:, s] for s in range(S)) + write[t] * y
                     for t in range(S)], axis=1)


def layer(cfg, W, i, X, latents):
    """latents: {layer: its latent rows}, filled and read here."""
    L, p, eps = cfg["layers"][i], f"l{i}.", cfg["norm"]["eps"]
    mx = L["mixer"]

    def sublayer(q, X, fn):
        hc = f"{p}hc{q}."
        h = rms_norm(read_streams(X, W[hc + "in"]), W[f"{p}norm{q}"], eps)
        return write_streams(X, fn(h), W[hc + "mix"], W[hc + "out"])

    def mixer(h):
        if L["type"] == "attention":
            return chunked_attention(h, W, p + "mix.", mx, eps)
        if L["type"] == "channel_delta":
            return delta_mixer(h, W, p + "mix.", mx, eps)
        src = mx.get("kv_from")
        if src is None:
            src = i
            latents[i] = latent_rows(h, W, p + "mix.", mx, eps)
        return latent_attention(h, W, p + "mix.", mx, eps, latents[src])

    X = sublayer(1, X, mixer)
    if L.get("mlp") is not None:
        X = sublayer(2, X, lambda h: dense_feed_forward(h, W, p + "mlp."))
    return X


def forward(cfg, W, tokens, capture=None):
    """Logits [n, vocab]; capture (a list) receives the sum of the streams
    after every layer."""
    X = np.repeat(W["embed"][np.asarray(tokens)][:, None], cfg.get("streams", 1), axis=1)
    latents = {}
    for i in range(len(cfg["layers"])):
        X = layer(cfg, W, i, X, latents)
        if capture is not None:
            capture.append(X.sum(1))
    return rms_norm(X.sum(1), W["final.norm"], cfg["norm"]["eps"]) @ W["head"].T


# ---------------------------------------------------------------------------
# weights for tests
# ---------------------------------------------------------------------------
def random_weights(cfg, seed, low_rank=5):
    """{name: bfloat16 torch tensor} for a config."""
    import torch

    rng = torch.Generator().manual_seed(seed)
    W = {}

    def mat(name, n_out, n_in, gain=1.0):
        W[name] = (torch.randn(n_out, n_in, generator=rng) * gain * n_in ** -0.5).bfloat16()

    def vec(name, n, center, spread=0.2):
        W[name] = (center + spread * torch.randn(n, generator=rng)).bfloat16()

    width, vocab, S = cfg["width"], cfg["vocab"], cfg.get("streams", 1)
    W["embed"] = torch.randn(vocab, width, generator=rng).bfloat16()
    mat("head", vocab, width, 2.0)
    vec("final.norm", width, 1.0)
    for i, L in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", L["mixer"]
        for q in (1, 2) if L.get("mlp") is not None else (1,):
            vec(f"{p}norm{q}", width, 1.0)
            hc = f"{p}hc{q}."
            vec(hc + "in", S, 1.0 / S, 0.4)
            vec(hc + "out", S, 1.0, 0.4)
            W[hc + "mix"] = (torch.eye(S) + 0.2 * torch.randn(S, S, generator=rng)).bfloat16()
        q = p + "mix."
        H, D, Dv = mx["heads"], mx["dim"], mx["vdim"]
        if L["type"] == "attention":
            G = mx["kv_heads"]
            for name, n in (("q", H * D), ("k", G * D), ("v", G * Dv)):
                mat(q + name, n, width)
                vec(f"{q}{name}.b", n, 0.0, 0.6)
            mat(q + "g", H, width, 2.0)
        elif L["type"] == "channel_delta":
            G, taps = mx["kv_heads"], mx["conv"]
            for name, n in (("q", G * D), ("k", G * D), ("v", H * Dv)):
                mat(q + name, n, width, 2.0)
                W[f"{q}{name}.conv"] = (0.6 * torch.randn(n, taps, generator=rng)).bfloat16()
            mat(q + "b", H, width, 2.0)
            vec(q + "A_log", H, -0.5, 1.0)
            vec(q + "norm", Dv, 1.0)
            mat(q + "a1", low_rank, width)
            mat(q + "a2", H * D, low_rank, 2.0)
            vec(q + "dt_bias", H * D, 0.0, 1.0)
            mat(q + "g1", low_rank + 2, width)
            mat(q + "g2", H * Dv, low_rank + 2, 2.0)
        else:
            R, Dr, Q = mx["kv_rank"], mx["rot_dim"], mx["q_rank"]
            mat(q + "dq", Q, width)
            vec(q + "dq.norm", Q, 1.0)
            mat(q + "uq", H * (D + Dr), Q, 2.0)
            if mx.get("kv_from") is None:
                mat(q + "dkv", R + Dr, width, 2.0)
                vec(q + "dkv.norm", R, 1.0)
            mat(q + "uk", H * D, R, 2.0)
            mat(q + "uv", H * Dv, R)
        mat(q + "o", width, H * Dv)
        if L.get("mlp") is not None:
            q, ff = p + "mlp.", L["mlp"]["ff"]
            for name in ("gate", "up"):
                mat(q + name, ff, width, 2.0)
                vec(f"{q}{name}.b", ff, 0.0, 0.5)
            mat(q + "down", width, ff)
            vec(q + "down.b", width, 0.0, 0.5)
    return W


def as_float64(W):
    return {k: v.double().numpy() for k, v in W.items()}
