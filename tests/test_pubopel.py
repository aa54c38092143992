"""Pubopel (dynamic tanh on both sides of every sublayer, input convolutions
with carried tails, attention whose values are its keys, with whole-projection
norms, score multipliers, a tanh cap, a distance bias, a sink and a window
behind which the first tokens stay visible, experts that read the token times
their sigmoid score) in the engine against the plain oracle in
pubopel_oracle.py: every mechanism alone, prompt vs token-by-token decoding,
prompt portions down to two tokens, unequal batches, reuse of freed cache
blocks and state slots, keys far back, at page borders and on both sides of
every window edge (planted so that one score stands out), first tokens, long
decoding, other sizes, and greedy generation through the engine's own
scheduler. CPU runs use the torch reference ops; the same cases run on the GPU
kernels under the gpu marker, where the kernels are also compared one by one
with the reference ops.
"""
import json
import os

import numpy as np
import pytest
import torch
from safetensors.torch import save_file

import pubopel_oracle as oracle
from kubeai_amd.engine import EngineConfig, LLMEngine, SamplingParams
from kubeai_amd.ops import seq as sops

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
GPU = [pytest.param("cuda", marks=pytest.mark.gpu)]


def moe(experts=5, top=2, ff=12, shared=10):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def att(heads=4, kv=2, dim=6, scale=0.4, softcap=3.0, mask=(11, 2), mlp=moe()):
    mx = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": scale}
    if softcap:
        mx["softcap"] = softcap
    if mask:
        mx["mask"] = {"size": mask[0], "keep_first": mask[1]}
    return {"type": "attention", "mixer": mx, "mlp": mlp}


def config(layers, width=24, vocab=40, eps=1e-5, taps=3):
    return {"architecture": "Pubopel", "vocab": vocab, "width": width,
            "norm": {"eps": eps}, "canon": {"taps": taps}, "layers": layers}


MIXED = config([att(), att(heads=3, kv=1, dim=4, mask=None, mlp=moe(3, 1)),
                att(heads=2, kv=2, dim=10, scale=0.3, softcap=None, mask=(5, 1)),
                att(mask=(19, 0), mlp=None)])


def model_dir(tmp_path, cfg, seed=0, W=None):
    d = str(tmp_path / ("m%d" % seed))
    os.makedirs(d, exist_ok=True)
    W = W if W is not None else oracle.random_weights(cfg, seed)
    with open(os.path.join(d, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in W.items()},
              os.path.join(d, "model.safetensors"))
    return d, oracle.as_float64(W)


def engine(d, device, dtype="float32", blocks=64, seqs=4):
    return LLMEngine(EngineConfig(
        model=d, device=device, dtype=dtype, num_gpu_blocks=blocks,
        max_num_seqs=seqs, max_model_len=1 << 20, max_num_batched_tokens=1 << 20,
        enable_prefix_caching=False, enable_graphs=False))


def tokens(n, vocab, seed):
    g = torch.Generator().manual_seed(9000 + seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def npy(t):
    return t.detach().double().cpu().numpy()


def check(got, want, dtype="float32", loose=0.25):
    got = npy(got) if isinstance(got, torch.Tensor) else got
    err = (np.abs(got - want).max(-1) / want.std()).max()
    # bf16: the widths here are tiny, so roundings do not average out
    assert err < (3e-4 if dtype == "float32" else loose), f"relative error {err:.3g}"


def replay(eng, rid, toks, cuts):
    """Feed toks in portions of the given sizes (the last repeats), wanting
    every position; returns [T, vocab]."""
    rows, at, i = [], 0, 0
    while at < len(toks):
        n = min(cuts[min(i, len(cuts) - 1)], len(toks) - at)
        part = toks[at : at + n]
        at += n
        i += 1
        out = eng.step_fixed([(rid, part, list(range(n)))],
                             [rid] if at == len(toks) else [])
        rows.append(out[0])
    return torch.cat(rows)


def meta_of(runs, positions, device, tables=None):
    return sops.SeqMeta.build(runs, torch.tensor(positions, dtype=torch.int32, device=device),
                              device, block_tables=tables)


# ---------------------------------------------------------------------------
# mechanisms as functions: the product's ops against the oracle's
# ---------------------------------------------------------------------------
def _dyt_params(C, g):
    return (torch.rand(1, generator=g) + 0.3, torch.randn(C, generator=g),
            torch.randn(C, generator=g))


def _dyt_np(x, p):
    return oracle.dyt(x, {"n.alpha": npy(p[0]), "n": npy(p[1]), "n.b": npy(p[2])}, "n")


def _on(p, device):
    return tuple(t.to(device) for t in p)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("C,taps", [(12, 3), (7, 4), (20, 1), (8, 2), (5, 9), (16, 16)])
def test_dyt_bracket_and_convolution_carry_their_state(device, C, taps):
    """The same tokens in one call and in portions of several sizes, over a
    slot that holds another sequence's tail."""
    g = torch.Generator().manual_seed(C * 100 + taps)
    T = 45
    post, pre = _dyt_params(C, g), _dyt_params(C, g)
    cw = 0.5 * torch.randn(C, taps, generator=g)
    res, br = torch.randn(T, C, generator=g), 2.0 * torch.randn(T, C, generator=g)
    new = npy(res) + _dyt_np(npy(br), post)
    want = oracle.input_convolution(_dyt_np(new, pre), npy(cw))
    for cuts in ([T], [1] * T, [17, 1, 2, 1, 24], [2] * 22 + [1], [33, 12], [4, 41]):
        tails = torch.full((3, taps - 1, C), 9.0, device=device)
        at, got, got_res = 0, [], []
        for n in cuts:
            meta = meta_of([(n, 1)], list(range(at, at + n)), device)
            o, r = sops.add_dyt_conv(br[at : at + n].to(device), _on(post, device),
                                     res[at : at + n].to(device), _on(pre, device),
                                     cw.to(device), tails, meta, torch.float32)
            got.append(o)
            got_res.append(r)
            at += n
        assert np.abs(npy(torch.cat(got_res)) - new).max() < 1e-5
        assert np.abs(npy(torch.cat(got)) - want).max() < 2e-5, cuts
        assert float((tails[0] - 9.0).abs().sum() + (tails[2] - 9.0).abs().sum()) == 0.0


@pytest.mark.parametrize("device", DEVICES)
def test_dyt_bracket_in_a_batch_of_unequal_runs(device):
    """Runs that start, end and lie inside the kernel's spans of tokens; one
    without a slot; the first call has no branch."""
    g = torch.Generator().manual_seed(3)
    C, taps = 12, 4
    post, pre = _dyt_params(C, g), _dyt_params(C, g)
    cw = 0.5 * torch.randn(C, taps, generator=g)
    lens = [1, 2, 37, 1, 3, 16, 5, 700, 2, 1]
    slots = [4, 0, 3, 7, 1, 2, -1, 5, 6, 8]
    tails = torch.full((9, taps - 1, C), 9.0, device=device)
    seqs = [torch.randn(n + 6, C, generator=g) for n in lens]
    at = [0] * len(lens)
    for step, sizes in enumerate((lens, [2, 1, 1, 3, 1, 1, 1, 1, 2, 1], [1] * 10, [3, 4, 1, 2, 4, 4, 4, 4, 2, 4])):
        runs, pos, rows = [], [], []
        for i, n in enumerate(sizes):
            n = min(n, len(seqs[i]) - at[i])
            runs.append((n, slots[i]))
            pos += range(at[i], at[i] + n)
            rows.append(seqs[i][at[i] : at[i] + n])
        res = torch.cat(rows)
        br = None if step == 0 else torch.zeros_like(res)
        zero = (post[0], post[1], torch.zeros(C))
        o, r = sops.add_dyt_conv(None if br is None else br.to(device),
                                 None if br is None else _on(zero, device), res.to(device),
                                 _on(pre, device), cw.to(device), tails,
                                 meta_of(runs, pos, device), torch.float32)
        assert np.abs(npy(r) - npy(res)).max() == 0.0
        s = 0
        for i, (n, slot) in enumerate(runs):
            h = _dyt_np(npy(seqs[i][: at[i] + n]), pre)
            if slot < 0:  # nothing is carried: earlier tokens count as zeros
                h[: at[i]] = 0.0
            want = oracle.input_convolution(h, npy(cw))[at[i] :]
            assert np.abs(npy(o[s : s + n]) - want).max() < 2e-5, (step, i)
            s += n
            at[i] += n


@pytest.mark.parametrize("device", DEVICES)
def test_final_norm_has_no_convolution(device):
    g = torch.Generator().manual_seed(8)
    post, pre = _dyt_params(10, g), _dyt_params(10, g)
    res, br = torch.randn(33, 10, generator=g), torch.randn(33, 10, generator=g)
    meta = meta_of([(33, 0)], list(range(33)), device)
    o, _ = sops.add_dyt_conv(br.to(device), _on(post, device), res.to(device),
                             _on(pre, device), None, None, meta, torch.float32)
    want = _dyt_np(npy(res) + _dyt_np(npy(br), post), pre)
    assert np.abs(npy(o) - want).max() < 1e-5


@pytest.mark.parametrize("device", DEVICES)
def test_dynamic_tanh_over_the_whole_range(device):
    """Tiny arguments (where 1 - e^-2x cancels), the seam between the kernel's
    two forms, saturation."""
    x = torch.cat([torch.logspace(-7, 2, 200), torch.linspace(0.24, 0.26, 50)])
    x = torch.cat([x, -x, torch.zeros(4)]).view(-1, 4)
    one = torch.ones(1), torch.ones(4), torch.zeros(4)
    meta = meta_of([(x.shape[0], 0)], list(range(x.shape[0])), device)
    o, _ = sops.add_dyt_conv(None, None, x.to(device), _on(one, device), None, None, meta,
                             torch.float32)
    want = np.tanh(npy(x))
    assert (np.abs(npy(o) - want) <= 6e-7 * np.abs(want)).all()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D", [(4, 2, 6), (3, 3, 8), (6, 1, 5), (1, 1, 16)])
def test_query_norm_and_cached_rows(device, H, G, D):
    """The cached row is the projected key; it and the number beside it give
    the normed key, with the weights folded into the query."""
    from kubeai_amd.models.mixers import TiedValueAttention

    g = torch.Generator().manual_seed(H * 10 + D)
    T, bs, eps = 9, 4, 1e-4
    qk = torch.randn(T, (H + G) * D + 3, generator=g)  # strided rows
    qn, kn = torch.randn(H * D, generator=g), torch.randn(G * D, generator=g)
    temp = torch.randn(H, generator=g)
    mx = TiedValueAttention(8, H, G, D, 1.0)
    w = mx.fold_query_weight(qn, kn, temp)
    cache = torch.zeros(6, G, bs, D, device=device)
    ks = torch.zeros(6, bs, 1, device=device)
    slots = torch.tensor([5, 4, 23, -1, 0, 1, 2, 3, 11], dtype=torch.int64)
    buf = qk.to(device).clone()
    q = buf[:, : H * D].unflatten(-1, (H, D))
    k = buf[:, H * D : (H + G) * D].unflatten(-1, (G, D))
    sops.qnorm_rows_to_cache(q, k, w.to(device), eps, cache, ks, slots.to(device))
    q0, k0 = npy(qk[:, : H * D]), npy(qk[:, H * D : (H + G) * D])
    qw = oracle.row_rms_norm(q0, npy(qn), eps).reshape(T, H, D) * npy(temp)[:, None]
    kw = oracle.row_rms_norm(k0, npy(kn), eps).reshape(T, G, D)
    assert np.abs(npy(buf[:, H * D :]) - npy(qk[:, H * D :])).max() == 0.0
    for t, s in enumerate(slots.tolist()):
        if s < 0:
            continue
        row, r = npy(cache[s // bs, :, s % bs]), float(ks[s // bs, s % bs, 0])
        assert np.abs(row - k0[t].reshape(G, D)).max() < 1e-6
        for u in range(T):
            for h in range(H):
                got = float(npy(q[u, h]) @ row[h // (H // G)]) * r
                want = float(qw[u, h] @ kw[t, h // (H // G)])
                assert abs(got - want) < 1e-4 * max(1.0, abs(want))
    used = {s for s in slots.tolist() if s >= 0}
    assert all(float(ks.view(-1)[s]) == 0.0 for s in range(24) if s not in used)


def _attend(device, q, rows, r, cuts, *, scale=0.5, softcap=0.0, window=0, keep=0,
            slopes=None, sink=None, block=16, dtype=torch.float32):
    """q [T, H, D] and rows [T, G, D] (keys and values, with a scale r [T] per
    key) through the paged attention op in portions; the blocks of the one
    sequence lie scattered."""
    T, H, D = q.shape
    G = rows.shape[1]
    nblk = (T + block - 1) // block
    perm = torch.randperm(nblk + 3, generator=torch.Generator().manual_seed(T)).tolist()
    table = torch.tensor([perm[:nblk]], dtype=torch.int32, device=device)
    cache = torch.zeros(nblk + 3, G, block, D, device=device, dtype=dtype)
    ks = torch.zeros(nblk + 3, block, 1, device=device)
    blk = torch.tensor(perm)[torch.arange(T) // block].to(device)
    off = (torch.arange(T) % block).to(device)
    outs, at = [], 0
    to = lambda t: None if t is None else t.to(device)
    for n in cuts:
        n = min(n, T - at)
        sl = slice(at, at + n)
        cache[blk[sl], :, off[sl]] = rows[sl].to(device, dtype)
        ks[blk[sl], off[sl], 0] = r[sl].to(device)
        meta = meta_of([(n, 0)], list(range(at, at + n)), device, table)
        out = torch.zeros(n, H, D, device=device, dtype=dtype)
        sops.masked_paged_attention(
            q[sl].to(device, dtype).contiguous(), cache, cache, meta, scale, out,
            softcap=softcap, window=window, keep_first=keep, slopes=to(slopes),
            key_scale=ks, sink=to(sink))
        outs.append(out)
        at += n
        if at >= T:
            break
    return torch.cat(outs)


def _attend_np(q, rows, r, *, scale=0.5, softcap=0.0, window=0, keep=0, slopes=None,
               sink=None):
    T, H, D = q.shape
    G = rows.shape[1]
    seen = oracle.visible_keys(T, {"size": window, "keep_first": keep} if window else None)
    out = np.zeros((T, H, D))
    for h in range(H):
        v = npy(rows[:, h // (H // G)])
        out[:, h] = oracle.head_attention(
            npy(q[:, h]), v * npy(r)[:, None], v, scale, 1.0, softcap,
            0.0 if slopes is None else float(slopes[h]),
            -np.inf if sink is None else float(sink[h]), seen)
    return out


FEATURES = {
    "plain": {},
    "window": dict(window=13),
    "kept": dict(window=13, keep=3),
    "kept_many": dict(window=5, keep=40),
    "window_one": dict(window=1, keep=1),
    "window_wide": dict(window=500, keep=2),
    "cap": dict(softcap=2.0),
    "bias": dict(slopes=True),
    "bias_kept": dict(slopes=True, window=9, keep=4),
    "sink": dict(sink=True),
    "all": dict(window=21, keep=5, softcap=3.0, slopes=True, sink=True),
}


def _features(name, H, seed):
    g = torch.Generator().manual_seed(seed)
    kw = dict(FEATURES[name])
    if kw.get("slopes"):
        kw["slopes"] = torch.tensor([oracle.head_slope(h, H) for h in range(H)])
    if kw.get("sink"):
        kw["sink"] = torch.randn(H, generator=g)
    return kw


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", sorted(FEATURES))
@pytest.mark.parametrize("H,G,D", [(4, 2, 6), (3, 3, 8)])
def test_attention_mask_bias_cap_sink(device, name, H, G, D):
    g = torch.Generator().manual_seed(H + D)
    T = 75
    q, rows = torch.randn(T, H, D, generator=g), torch.randn(T, G, D, generator=g)
    r = torch.rand(T, generator=g) + 0.3
    kw = _features(name, H, 1)
    want = _attend_np(q, rows, r, **kw)
    for cuts in ([T], [1] * T, [20, 1, 2, 1, 51]):
        got = npy(_attend(device, q, rows, r, cuts, **kw))
        assert np.abs(got - want).max() < 2e-5, cuts


@pytest.mark.parametrize("device", GPU)
@pytest.mark.parametrize("name", sorted(FEATURES))
@pytest.mark.parametrize("H,G,D", [(8, 2, 128), (8, 2, 64), (4, 2, 64), (4, 1, 48), (16, 1, 96),
                                   (20, 1, 32), (4, 4, 16), (5, 1, 144), (8, 1, 256),
                                   (2, 1, 320)])
def test_attention_matrix_core_kernels(device, name, H, G, D):
    g = torch.Generator().manual_seed(H + D)
    T = 150
    q, rows = (torch.randn(T, n, D, generator=g).bfloat16().float() for n in (H, G))
    r = torch.rand(T, generator=g) + 0.3
    kw = _features(name, H, 1)
    want = _attend_np(q, rows, r, scale=D ** -0.5, **kw)
    for cuts in ([T], [100, 1, 1, 48], [T - 20] + [1] * 20):
        got = npy(_attend(device, q, rows, r, cuts, scale=D ** -0.5, dtype=torch.bfloat16,
                          **kw).float())
        assert np.abs(got - want).max() < 0.03, cuts


@pytest.mark.parametrize("device", GPU)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_attention_long_batch_with_splits(device, dtype):
    """Contexts long enough that decoded keys are split over blocks, sequences
    of unequal length, block size 32 and one that is no power of two."""
    g = torch.Generator().manual_seed(4)
    H, G, D = 8, 2, 64
    for bs in (32, 24):
        lens = [1500, 3, 700, 65, 1]
        total = sum((n + bs - 1) // bs for n in lens)
        cache = torch.randn(total, G, bs, D, generator=g).to(dtype)
        ks = torch.rand(total, bs, 1, generator=g) + 0.3
        perm = torch.randperm(total, generator=g)
        table = torch.zeros(len(lens), max((n + bs - 1) // bs for n in lens), dtype=torch.int32)
        s = 0
        for i, n in enumerate(lens):
            k = (n + bs - 1) // bs
            table[i, :k] = perm[s : s + k].int()
            s += k
        q = torch.randn(len(lens), H, D, generator=g).to(dtype)
        kw = _features("all", H, 2)
        kw2 = dict(softcap=kw["softcap"], slopes=kw["slopes"] * 0.05, sink=kw["sink"])
        for extra in ({}, dict(window=600, keep_first=9)):
            meta = meta_of([(1, i) for i in range(len(lens))], [n - 1 for n in lens], "cpu", table)
            want = torch.zeros(len(lens), H, D)
            sops.masked_paged_attention(q.float(), cache.float(), cache.float(), meta, D ** -0.5,
                                        want, key_scale=ks, **kw2, **extra)
            meta = meta_of([(1, i) for i in range(len(lens))], [n - 1 for n in lens], device,
                           table.to(device))
            out = torch.zeros(len(lens), H, D, dtype=dtype, device=device)
            c = cache.to(device)
            sops.masked_paged_attention(
                q.to(device), c, c, meta, D ** -0.5, out, key_scale=ks.to(device),
                **{k: v.to(device) if isinstance(v, torch.Tensor) else v for k, v in kw2.items()},
                **extra)
            tol = 2e-5 if dtype == torch.float32 else 0.02
            assert float((out.float().cpu() - want).abs().max()) < tol


def test_kept_tokens_and_chunks_do_not_combine():
    q = torch.zeros(1, 1, 4)
    with pytest.raises(ValueError):
        sops.masked_paged_attention(q, None, None, None, 1.0, q, chunk=4, keep_first=1)


# query, key, is it visible behind a window of 40 that keeps 6
EDGES = [(99, 60, True), (99, 59, False), (100, 61, True), (100, 60, False), (47, 8, True),
         (47, 7, False), (47, 5, True), (47, 6, False), (700, 0, True), (700, 5, True),
         (700, 6, False), (700, 661, True), (700, 660, False), (1029, 990, True),
         (1029, 989, False), (45, 6, True), (46, 6, False), (16, 0, True), (15, 15, True),
         (39, 0, True), (40, 5, True)]


def _planted(device, q_pos, key_pos, decode, dims=(2, 1, 8), dtype=torch.float32, boost=40.0):
    """Random keys, but the key at key_pos and the query at q_pos are aligned
    and long: visible, it takes all the weight."""
    H, G, D = dims
    T = q_pos + 1
    g = torch.Generator().manual_seed(q_pos * 31 + key_pos)
    q, rows = 0.2 * torch.randn(T, H, D, generator=g), 0.3 * torch.randn(T, G, D, generator=g)
    r = torch.ones(T)
    rows[key_pos, 0] = 0.0
    rows[key_pos, 0, 1] = boost
    q[q_pos, :, 1] = 1.0
    q, rows = (x.to(dtype).float() for x in (q, rows))
    kw = dict(scale=1.0, window=40, keep=6, softcap=60.0,
              slopes=torch.full((H,), 1e-3), sink=torch.zeros(H))
    cuts = [q_pos, 1] if decode and q_pos else [T]
    got = npy(_attend(device, q, rows, r, cuts, dtype=dtype, **kw).float())[q_pos]
    want = _attend_np(q, rows, r, **kw)[q_pos]
    return got, want, boost


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("q_pos,key_pos,seen", EDGES)
def test_planted_key_at_every_edge(device, decode, q_pos, key_pos, seen):
    got, want, boost = _planted(device, q_pos, key_pos, decode)
    assert (want[0, 1] > 0.9 * boost) == seen
    assert np.abs(got - want).max() < 1e-3


@pytest.mark.parametrize("device", GPU)
@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("dims", [(8, 2, 64), (4, 1, 128), (16, 1, 32), (4, 2, 64)])
@pytest.mark.parametrize("q_pos,key_pos,seen", EDGES)
def test_planted_key_matrix_core_kernels(device, decode, dims, q_pos, key_pos, seen):
    got, want, boost = _planted(device, q_pos, key_pos, decode, dims=dims, dtype=torch.bfloat16)
    assert (want[0, 1] > 0.9 * boost) == seen
    assert np.abs(got - want).max() < (0.2 if seen else 0.03)


@pytest.mark.parametrize("device", DEVICES)
def test_sink_share_at_known_scores(device):
    """Equal scores s over n keys and values of one: the output is
    n e^s / (n e^s + e^sink), the sink neither scaled, capped nor biased."""
    n, H = 7, 3
    q, rows = torch.zeros(n, H, 4), torch.ones(n, 1, 4)
    sink = torch.tensor([0.0, 1.5, -20.0])
    got = npy(_attend(device, q, rows, torch.ones(n), [n], scale=7.0, softcap=2.0, sink=sink))
    for h in range(H):
        want = n / (n + np.exp(float(sink[h])))
        assert np.abs(got[n - 1, h] - want).max() < 1e-6


@pytest.mark.parametrize("device", DEVICES)
def test_sigmoid_scores_and_weighted_input(device):
    z = torch.tensor([[0.1, 2.0, -1.0, 2.0, 0.5], [-3.0, -3.5, -9.0, -4.0, -3.2]])
    dense, w, idx = sops.router_scores_topk(z.to(device), 2, None, 1.0, "sigmoid")
    s = oracle.sigmoid(npy(z))
    assert idx.cpu().tolist() == [[1, 3], [0, 4]]  # ties: the lower index first
    for t in range(2):
        for j, e in enumerate(idx.cpu()[t].tolist()):
            assert abs(float(w[t, j]) - s[t, e]) < 1e-6
            assert abs(float(dense[t, e]) - s[t, e]) < 1e-6
    assert int((dense > 0).sum()) == 4
    # the weight goes in before the activation, for both factors
    g = torch.Generator().manual_seed(5)
    gu, rw = 2.0 * torch.randn(6, 2 * 3 * 8, generator=g), torch.rand(6, 3, generator=g)
    rw[2, 1] = 0.0
    got = npy(sops.glu_weighted(gu.to(device), rw.to(device), 8, w_input=True))
    a = npy(gu).reshape(6, 3, 2, 8) * npy(rw)[:, :, None, None]
    want = (a[:, :, 0] * oracle.sigmoid(a[:, :, 0]) * a[:, :, 1]).reshape(6, 24)
    assert np.abs(got - want).max() < 1e-5
    assert np.abs(got[2, 8:16]).max() == 0.0


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("T", [7, 300])  # every expert's product; gathered tokens
@pytest.mark.parametrize("experts,top,shared", [(5, 2, 10), (3, 1, 0), (4, 4, 6), (1, 1, 4)])
def test_routed_feed_forward(device, T, experts, top, shared):
    from kubeai_amd.models.mixers import RoutedGatedMoE

    mlp = moe(experts, top, 12, shared)
    W = oracle.as_float64(oracle.random_weights(config([att(mlp=mlp)]), 17))
    m = RoutedGatedMoE(24, experts, top, 12, correction=False, shared_ff=shared,
                       score="sigmoid", weight_on="input").to(device)
    pre = "l0.mlp."
    names = [f"{pre}e{e}." for e in range(experts)] + ([pre + "shared."] if shared else [])
    t = lambda a: torch.tensor(a, dtype=torch.float32)
    m.gate_up.weight.data.copy_(torch.cat([t(W[n + x]) for n in names for x in ("gate", "up")]))
    m.down.weight.data.copy_(torch.cat([t(W[n + "down"]) for n in names], 1))
    m.router.data.copy_(t(W[pre + "router"]))
    h = torch.randn(T, 24, generator=torch.Generator().manual_seed(T))
    with torch.inference_mode():
        got = npy(m(h.to(device)))
    want = oracle.routed_ff(npy(h), W, pre, mlp)
    assert np.abs(got - want).max() < 2e-4 * max(1.0, np.abs(want).max())


# ---------------------------------------------------------------------------
# the engine against whole-sequence oracle runs
# ---------------------------------------------------------------------------
SINGLE = {
    "attention": config([att(mlp=None)]),
    "attention_moe": config([att()]),
    "full_attention": config([att(mask=None, mlp=None)]),
    "no_cap": config([att(softcap=None, mlp=None)]),
    "two_layers": config([att(mlp=None), att(heads=2, kv=1, mask=(4, 3), mlp=None)]),
    "one_tap": config([att()], taps=1),
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", sorted(SINGLE))
def test_each_mechanism_whole_prompt(tmp_path, device, name):
    cfg = SINGLE[name]
    d, W = model_dir(tmp_path, cfg, seed=1)
    toks = tokens(29, cfg["vocab"], 1)
    check(replay(engine(d, device), "a", toks, [len(toks)]), oracle.forward(cfg, W, toks))


@pytest.mark.parametrize("device", DEVICES)
def test_residual_after_every_layer(tmp_path, device):
    d, W = model_dir(tmp_path, MIXED, seed=2)
    toks = tokens(21, MIXED["vocab"], 2)
    eng = engine(d, device)
    eng.runner.model.capture_layers = []
    replay(eng, "a", toks, [len(toks)])
    want = []
    oracle.forward(MIXED, W, toks, want)
    got = eng.runner.model.capture_layers
    assert len(got) == len(want) == len(MIXED["layers"])
    for i, (a, b) in enumerate(zip(got, want)):
        a = npy(a)[: len(toks)]  # a step may be padded to a bucket
        assert np.abs(a - b).max() < 2e-4 * max(1.0, np.abs(b).max()), i


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cuts", [[1], [2], [3, 2, 5], [7, 1, 1, 4, 1], [16, 1], [11, 13]])
def test_portions_and_token_by_token(tmp_path, device, cuts):
    d, W = model_dir(tmp_path, MIXED, seed=3)
    toks = tokens(38, MIXED["vocab"], 3)
    check(replay(engine(d, device), "a", toks, cuts), oracle.forward(MIXED, W, toks))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("n", [1, 2, 3])
def test_first_tokens(tmp_path, device, n):
    d, W = model_dir(tmp_path, MIXED, seed=4)
    toks = tokens(n, MIXED["vocab"], 4)
    want = oracle.forward(MIXED, W, toks)
    check(replay(engine(d, device), "a", toks, [n]), want)
    check(replay(engine(d, device), "b", toks, [1]), want)


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding(tmp_path, device):
    """Windows of every layer pass over decoded tokens."""
    cfg = config([att(), att(mask=(30, 1), mlp=None)])
    d, W = model_dir(tmp_path, cfg, seed=5)
    toks = tokens(110, cfg["vocab"], 5)
    check(replay(engine(d, device), "a", toks, [6, 1]), oracle.forward(cfg, W, toks))


@pytest.mark.parametrize("device", DEVICES)
def test_long_prompt_in_one_step_and_routed_path(tmp_path, device):
    """More than 256 tokens in a step take the per-expert gather path of the
    routed feed-forward; the same prompt in portions takes the dense one."""
    cfg = config([att(), att(mask=None)])
    d, W = model_dir(tmp_path, cfg, seed=6)
    toks = tokens(300, cfg["vocab"], 6)
    want = oracle.forward(cfg, W, toks)
    check(replay(engine(d, device), "a", toks, [300]), want)
    check(replay(engine(d, device), "b", toks, [270, 2, 1]), want)


OTHER = {
    # values that are equal or 1 in one place differ or are larger in another
    "every_head_its_own_key": config([att(heads=3, kv=3, dim=8)]),
    "one_head": config([att(heads=1, kv=1, dim=4)]),
    "one_key_head": config([att(heads=6, kv=1, dim=2)]),
    "window_of_one": config([att(mask=(1, 0)), att(mask=(1, 4))]),
    "keep_more_than_window": config([att(mask=(3, 9))]),
    "keep_one": config([att(mask=(6, 1))]),
    "wide_window": config([att(mask=(200, 3))]),
    "top_one": config([att(mlp=moe(experts=3, top=1))]),
    "all_experts": config([att(mlp=moe(experts=3, top=3))]),
    "one_expert": config([att(mlp=moe(experts=1, top=1))]),
    "no_shared_expert": config([att(mlp=moe(shared=None))]),
    "two_taps": config([att()], taps=2),
    "six_taps": config([att(), att()], taps=6),
    "small_cap": config([att(softcap=0.5, scale=2.0)]),
    "sixteens": config([att(heads=4, kv=1, dim=32, scale=0.2, mask=(18, 3), mlp=moe(4, 2, 16, 48)),
                        att(heads=4, kv=2, dim=16, scale=0.25, mask=None, mlp=moe(3, 1, 32, 16))],
                       width=64, vocab=80),
    "odd_width": config([att(), att(mask=None)], width=23),
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", sorted(OTHER))
def test_other_sizes(tmp_path, device, name):
    cfg = OTHER[name]
    d, W = model_dir(tmp_path, cfg, seed=7)
    toks = tokens(26, cfg["vocab"], 7)
    check(replay(engine(d, device), "a", toks, [9, 2, 1]), oracle.forward(cfg, W, toks))


@pytest.mark.parametrize("device", GPU)
@pytest.mark.parametrize("name", ["sixteens", "odd_width", "keep_more_than_window"])
def test_bfloat16_serving_precision(tmp_path, device, name):
    cfg = OTHER[name]
    d, W = model_dir(tmp_path, cfg, seed=8)
    toks = tokens(70, cfg["vocab"], 8)
    want = oracle.forward(cfg, W, toks)
    a = replay(engine(d, device, "bfloat16"), "a", toks, [70])
    b = replay(engine(d, device, "bfloat16"), "b", toks, [33, 2, 1])
    for got in (a, b):
        err = np.abs(npy(got) - want).max(-1) / want.std()
        # a rounding may flip a close routing decision of single tokens
        assert np.median(err) < 0.1 and (err > 0.4).mean() <= 0.1, (np.median(err), err.max())


@pytest.mark.parametrize("device", DEVICES)
def test_unequal_batch_matches_each_alone(tmp_path, device):
    d, W = model_dir(tmp_path, MIXED, seed=11)
    lens = {"a": 41, "b": 3, "c": 18, "d": 1}
    toks = {r: tokens(n, MIXED["vocab"], 10 + i) for i, (r, n) in enumerate(lens.items())}
    want = {r: oracle.forward(MIXED, W, t) for r, t in toks.items()}
    eng = engine(d, device)
    at = {r: 0 for r in toks}
    got = {r: [] for r in toks}
    plan = {"a": [5, 1, 1, 9, 2], "b": [1], "c": [2, 7, 1], "d": [1]}
    step = 0
    while any(at[r] < lens[r] for r in toks):
        entries, end = [], []
        for r in toks:
            if at[r] >= lens[r] or (r == "c" and step % 3 == 1):  # c sits some steps out
                continue
            n = min(plan[r][min(step, len(plan[r]) - 1)], lens[r] - at[r])
            entries.append((r, toks[r][at[r] : at[r] + n], list(range(n))))
            at[r] += n
            if at[r] == lens[r]:
                end.append(r)
        for (r, _, _), rows in zip(entries, eng.step_fixed(entries, end)):
            got[r].append(rows)
        step += 1
    for r in toks:
        check(torch.cat(got[r]), want[r])
    assert eng.block_manager.num_free_blocks == eng.block_manager.num_blocks


@pytest.mark.parametrize("device", DEVICES)
def test_freed_blocks_and_slots_are_reused(tmp_path, device):
    d, W = model_dir(tmp_path, MIXED, seed=12)
    eng = engine(d, device, blocks=5, seqs=2)  # 80 tokens, two state slots
    for i in range(4):
        ta, tb = tokens(40 + i, MIXED["vocab"], 20 + i), tokens(17, MIXED["vocab"], 40 + i)
        ra, rb = "a%d" % i, "b%d" % i
        out = eng.step_fixed([(ra, ta[:30], list(range(30))), (rb, tb[:2], [0, 1])])
        ga, gb = [out[0]], [out[1]]
        out = eng.step_fixed([(rb, tb[2:], list(range(15))), (ra, ta[30:31], [0])], [rb])
        gb.append(out[0])
        ga.append(out[1])
        out = eng.step_fixed([(ra, ta[31:], list(range(len(ta) - 31)))], [ra])
        ga.append(out[0])
        check(torch.cat(ga), oracle.forward(MIXED, W, ta))
        check(torch.cat(gb), oracle.forward(MIXED, W, tb))
    with pytest.raises(Exception):
        eng.step_fixed([("x", tokens(81, MIXED["vocab"], 0), [])])


@pytest.mark.parametrize("device", DEVICES)
def test_window_edge_and_kept_tokens_in_the_logits(tmp_path, device):
    """A one-layer model without convolution reach: the last position must
    ignore a change just outside its window and just behind the kept tokens,
    and follow the oracle for one just inside either."""
    n, size, keep = 60, 17, 4
    cfg = config([att(mask=(size, keep), mlp=None)], taps=1)
    d, W = model_dir(tmp_path, cfg, seed=31)
    base = tokens(n, cfg["vocab"], 31)
    eng = engine(d, device)

    def last(toks, rid):
        got = replay(eng, rid, toks, [n - 9, 2, 1])[-1:]
        check(got, oracle.forward(cfg, W, toks)[-1:])
        return npy(got)

    ref = last(base, "r")
    for pos, seen in ((n - size, True), (n - size - 1, False), (keep - 1, True), (keep, False)):
        toks = list(base)
        toks[pos] = (toks[pos] + 7) % cfg["vocab"]
        diff = np.abs(last(toks, "p%d" % pos) - ref).max()
        assert (diff > 1e-4) == seen, (pos, diff)


@pytest.mark.parametrize("device", DEVICES)
def test_far_token_reaches_logits(tmp_path, device):
    """Two prompts that differ in their first token only, hundreds of tokens
    before the last one: it stays visible as a kept token."""
    cfg = config([att(mask=(30, 2), mlp=None)])
    W = oracle.random_weights(cfg, 30)
    W["l0.mix.sink"] = torch.full_like(W["l0.mix.sink"], -3.0)
    d, W64 = model_dir(tmp_path, cfg, seed=30, W=W)
    base = tokens(420, cfg["vocab"], 30)
    other = [(base[0] + 1) % cfg["vocab"]] + base[1:]
    rows = []
    for rid, toks in (("x", base), ("y", other)):
        got = replay(engine(d, device, blocks=40), rid, toks, [400, 17, 1])
        want = oracle.forward(cfg, W64, toks)
        check(got[-4:], want[-4:])
        rows.append(want[-1])
    assert np.abs(rows[0] - rows[1]).max() > 1e-4 * rows[0].std()


def test_unconsumed_missing_and_odd_settings_are_errors(tmp_path):
    cfg = SINGLE["attention_moe"]
    W = oracle.random_weights(cfg, 0)
    d, _ = model_dir(tmp_path, cfg, seed=40, W=dict(W, **{"l0.mix.v": torch.zeros(3).bfloat16()}))
    with pytest.raises(ValueError, match="not consumed"):
        engine(d, "cpu")
    d, _ = model_dir(tmp_path, cfg, seed=41,
                     W={k: v for k, v in W.items() if k != "l0.norm2b.alpha"})
    with pytest.raises(ValueError, match="lacks"):
        engine(d, "cpu")
    bad = json.loads(json.dumps(cfg))
    bad["layers"][0]["mixer"]["vdim"] = 7  # the values are the keys
    d, _ = model_dir(tmp_path, bad, seed=42, W=W)
    with pytest.raises(ValueError, match="vdim"):
        engine(d, "cpu")
    from kubeai_amd.models.config import pubopel_arch_config
    with pytest.raises(ValueError):
        pubopel_arch_config(dict(cfg, canon={"taps": 0}))


def test_cache_keeps_one_row_and_one_number_per_token(tmp_path):
    d, _ = model_dir(tmp_path, SINGLE["attention"], seed=43)
    eng = engine(d, "cpu", blocks=7)
    rows, values, scales = eng.runner.kv_caches[0]
    assert rows.shape == (7, 2, 16, 6) and values.numel() == 0
    assert scales.shape == (7, 16, 1) and scales.dtype == torch.float32


# ---------------------------------------------------------------------------
# generation through the engine's own entry point and scheduler
# ---------------------------------------------------------------------------
def _generate(eng, prompts, max_tokens, arrive_every=0):
    pending = list(prompts.items())
    if not arrive_every:
        for rid, t in pending:
            eng.add_request(t, SamplingParams(max_tokens=max_tokens, ignore_eos=True),
                            request_id=rid)
        pending = []
    done, steps = {}, 0
    while (pending or eng.has_work()) and steps < 600:
        if pending and steps % arrive_every == 0:
            rid, t = pending.pop(0)
            eng.add_request(t, SamplingParams(max_tokens=max_tokens, ignore_eos=True),
                            request_id=rid)
        for o in eng.step():
            if o.finished:
                done[o.request_id] = list(o.output_token_ids)
        steps += 1
    return done


def _assert_greedy(cfg, W, prompts, done, tol):
    assert set(done) == set(prompts)
    for rid, t in prompts.items():
        gen = done[rid]
        logits = oracle.forward(cfg, W, t + gen)
        for i, tok in enumerate(gen):
            row = logits[len(t) - 1 + i]
            assert row[tok] >= row.max() - tol * row.std(), (rid, i)


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_scheduler(tmp_path, device):
    d, W = model_dir(tmp_path, MIXED, seed=20)
    eng = LLMEngine(EngineConfig(
        model=d, device=device, dtype="float32", num_gpu_blocks=40, max_num_seqs=3,
        max_model_len=256, max_num_batched_tokens=24,  # prompts get chunked
        enable_graphs=False))
    prompts = {"p%d" % i: tokens(n, MIXED["vocab"], 50 + i)
               for i, n in enumerate([31, 5, 47, 12, 2])}
    done = _generate(eng, prompts, 12)
    assert all(len(g) == 12 for g in done.values())
    _assert_greedy(MIXED, W, prompts, done, 1e-3)
    assert eng.block_manager.num_free_blocks == eng.block_manager.num_blocks


def test_requests_arriving_under_a_tight_pool(tmp_path):
    d, W = model_dir(tmp_path, MIXED, seed=21)
    eng = LLMEngine(EngineConfig(
        model=d, device="cpu", dtype="float32", num_gpu_blocks=7, max_num_seqs=2,
        max_model_len=128, max_num_batched_tokens=16, enable_graphs=False))
    prompts = {"q%d" % i: tokens(n, MIXED["vocab"], 60 + i) for i, n in enumerate([30, 9, 21, 4])}
    done = _generate(eng, prompts, 10, arrive_every=3)
    _assert_greedy(MIXED, W, prompts, done, 1e-3)
    assert eng.block_manager.num_free_blocks == eng.block_manager.num_blocks


@pytest.mark.gpu
def test_decode_graph_replays_match_oracle(tmp_path):
    cfg = OTHER["sixteens"]
    d, W = model_dir(tmp_path, cfg, seed=22)
    eng = LLMEngine(EngineConfig(
        model=d, device="cuda", dtype="float32", num_gpu_blocks=40, max_num_seqs=4,
        max_model_len=256, max_num_batched_tokens=64, enable_graphs=True))
    prompts = {"g%d" % i: tokens(n, cfg["vocab"], 70 + i) for i, n in enumerate([9, 20, 3])}
    done = _generate(eng, prompts, 24)
    assert all(len(g) == 24 for g in done.values())
    _assert_greedy(cfg, W, prompts, done, 1e-3)


@pytest.mark.gpu
def test_bfloat16_decode_graphs_follow_the_oracle(tmp_path):
    cfg = OTHER["sixteens"]
    d, W = model_dir(tmp_path, cfg, seed=23)
    eng = LLMEngine(EngineConfig(
        model=d, device="cuda", dtype="bfloat16", num_gpu_blocks=40, max_num_seqs=4,
        max_model_len=256, max_num_batched_tokens=64, enable_graphs=True))
    prompts = {"g%d" % i: tokens(n, cfg["vocab"], 80 + i) for i, n in enumerate([9, 20, 3, 33])}
    done = _generate(eng, prompts, 20)
    good = 0
    for rid, t in prompts.items():
        rows = oracle.forward(cfg, W, t + done[rid])[len(t) - 1 : -1]
        good += sum(r[tok] >= r.max() - 0.5 * r.std() for r, tok in zip(rows, done[rid]))
    assert good >= 0.9 * 20 * len(prompts)


def test_preset_builds_and_generates():
    eng = LLMEngine(EngineConfig(
        model="pubopel-tiny", device="cpu", dtype="float32", num_gpu_blocks=16,
        max_num_seqs=2, max_model_len=64, enable_graphs=False))
    done = _generate(eng, {"a": tokens(9, 512, 1), "b": tokens(3, 512, 2)}, 5)
    assert all(len(g) == 5 for g in done.values())


# ---------------------------------------------------------------------------
# kernels one by one against the reference ops
# ---------------------------------------------------------------------------
def _close(got, want, dtype):
    if want.numel() == 0:
        return
    tol = 2e-5 if dtype == torch.float32 else 2e-2
    scale = max(1.0, float(want.float().abs().max()))
    assert float((got.float().cpu() - want.float()).abs().max()) <= tol * scale


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("C,taps", [(24, 3), (1000, 4), (2048, 4), (36, 8), (64, 12), (7, 6), (64, 1)])
def test_kernel_dyt_conv(dtype, C, taps):
    g = torch.Generator().manual_seed(C)
    for lens, starts in (([70, 1, 19, 1, 2, 4], [0, 5, 0, 9, 33, 0]), ([1] * 9, list(range(9))),
                         ([5000], [3]), ([600], [0]), ([2, 2, 3], [0, 1, 2])):
        T = sum(lens)
        slots = [(3 * i + 1) % 10 if i != 3 else -1 for i in range(len(lens))]
        pos = [s + p for n, s in zip(lens, starts) for p in range(n)]
        post, pre = _dyt_params(C, g), _dyt_params(C, g)
        cw = 0.3 * torch.randn(C, taps, generator=g)
        res = torch.randn(T, C, generator=g)
        for br in (torch.randn(T, C, generator=g).to(dtype), torch.randn(T, C, generator=g), None):
            tails = torch.randn(10, taps - 1, C, generator=g)
            tc, tg = tails.clone(), tails.cuda()
            runs = list(zip(lens, slots))
            want, wr = sops.add_dyt_conv(br, post, res, pre, cw, tc, meta_of(runs, pos, "cpu"), dtype)
            got, gr = sops.add_dyt_conv(None if br is None else br.cuda(), _on(post, "cuda"),
                                        res.cuda(), _on(pre, "cuda"), cw.cuda(), tg,
                                        meta_of(runs, pos, "cuda"), dtype)
            _close(got, want, dtype)
            _close(gr, wr, torch.float32)
            _close(tg, tc, torch.float32)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D", [(16, 4, 128), (4, 2, 6), (8, 8, 64), (3, 1, 40)])
def test_kernel_qnorm_rows(dtype, H, G, D):
    g = torch.Generator().manual_seed(D)
    T = 21
    qk = torch.randn(T, (H + G) * D, generator=g).to(dtype)
    w = torch.randn(H * D, generator=g)
    slots = torch.randperm(64, generator=g)[:T]
    slots[3] = -1
    outs = []
    for device in ("cpu", "cuda"):
        buf = qk.to(device).clone()
        q = buf[:, : H * D].unflatten(-1, (H, D))
        k = buf[:, H * D :].unflatten(-1, (G, D))
        cache = torch.zeros(4, G, 16, D, dtype=dtype, device=device)
        ks = torch.zeros(4, 16, 1, device=device)
        sops.qnorm_rows_to_cache(q, k, w.to(device), 1e-6, cache, ks, slots.to(device))
        outs.append((buf, cache, ks))
    for a, b in zip(outs[1], outs[0]):
        _close(a, b, dtype)
    assert torch.equal(outs[1][1].cpu(), outs[0][1])


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("N,E", [(1, 1), (7, 3), (600, 5), (5000, 8), (300, 70), (2049, 2)])
def test_expert_order_is_a_stable_sort(device, N, E):
    top = 2 if N % 2 == 0 else 1
    g = torch.Generator().manual_seed(N)
    idx = torch.randint(0, E, (N // top, top), generator=g, dtype=torch.int32)
    if E == 3:
        idx[:] = 1  # experts without tokens
    w = torch.rand(N // top, top, generator=g)
    tok, wrow, place, counts = sops.expert_order(idx.to(device), w.to(device), E)
    order = np.argsort(idx.flatten().numpy(), kind="stable")
    assert tok.cpu().tolist() == (order // top).tolist()
    assert np.array_equal(wrow.cpu().numpy().ravel(), w.flatten().numpy()[order])
    inv = np.empty(N, dtype=int)
    inv[order] = np.arange(N)
    assert place.cpu().flatten().tolist() == inv.tolist()
    assert counts.cpu().tolist() == np.bincount(idx.flatten().numpy(), minlength=E).tolist()
    y, sh = torch.randn(N, 24, generator=g), torch.randn(N // top, 24, generator=g)
    want = npy(y)[inv].reshape(N // top, top, 24).sum(1)
    got = sops.combine_expert_rows(y.to(device), place, None)
    assert np.abs(npy(got) - want).max() < 1e-5
    got = sops.combine_expert_rows(y.to(device), place, sh.to(device))
    assert np.abs(npy(got) - want - npy(sh)).max() < 1e-5


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("T,C,E,extra,top", [(5, 24, 5, 0, 2), (1, 64, 8, 1, 1), (70, 1000, 8, 0, 2),
                                             (1500, 64, 3, 1, 3), (33, 40, 130, 0, 6), (9, 7, 1, 0, 1)])
def test_router_in_one_step(device, T, C, E, extra, top):
    """Logits, scores and choice from the activations: as plain products and
    a sort give them."""
    g = torch.Generator().manual_seed(T + C)
    h, R = torch.randn(T, C, generator=g), torch.randn(E + extra, C, generator=g) * C ** -0.5
    bias = 0.3 * torch.randn(E, generator=g)
    for score in ("softmax", "sigmoid"):
        for b in (None, bias):
            dense, w, idx, ex = sops.route_tokens(h.to(device), R.to(device), E, top,
                                                  None if b is None else b.to(device), 1.3, score)
            z = npy(h) @ npy(R).T
            e = np.exp(z[:, :E] - z[:, :E].max(-1, keepdims=True))
            s = oracle.sigmoid(z[:, :E]) if score == "sigmoid" else e / e.sum(-1, keepdims=True)
            key = s if b is None else s + npy(b)
            order = np.argsort(-key, axis=-1, kind="stable")[:, :top]
            assert np.array_equal(idx.cpu().numpy(), order)
            assert np.abs(npy(w) - np.take_along_axis(s, order, 1) * 1.3).max() < 1e-5
            want = np.zeros((T, E))
            np.put_along_axis(want, order, np.take_along_axis(s, order, 1) * 1.3, 1)
            assert np.abs(npy(dense) - want).max() < 1e-5
            if extra:
                assert np.abs(npy(ex) - z[:, E:]).max() < 1e-4
            else:
                assert ex is None


@pytest.mark.parametrize("device", DEVICES)
def test_router_ties_take_the_lower_expert(device):
    h = torch.ones(3, 8)
    R = torch.ones(70, 8) * 0.1
    R[65] = 0.2
    _, _, idx, _ = sops.route_tokens(h.to(device), R.to(device), 70, 3, None, 1.0, "sigmoid")
    assert idx.cpu().tolist() == [[65, 0, 1]] * 3
