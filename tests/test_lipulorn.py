"""Lipulorn (gated delta rule with a decay per key channel / windowed latent
attention whose cached rows several layers may share / chunk attention with
unit-RMS heads and head gates; residual streams; biased silu feed-forwards) in
the engine against the plain oracle in lipulorn_oracle.py: every mechanism
alone, prompt vs token-by-token decoding, prompt portions down to two tokens,
unequal batches, reuse of freed cache blocks and state slots, keys just inside
and just outside every window and chunk, at page borders and far back (planted
so that one score stands out), first tokens, long decoding, other sizes, and
greedy generation through the engine's own scheduler. CPU runs use the torch
reference ops; the same cases run on the GPU kernels under the gpu marker,
where the kernels are also compared one by one with the reference ops.
"""
import json
import os

import numpy as np
import pytest
import torch
from safetensors.torch import save_file

import lipulorn_oracle as oracle
from kubeai_amd.engine import EngineConfig, LLMEngine, SamplingParams
from kubeai_amd.ops import seq as sops

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
GPU = [pytest.param("cuda", marks=pytest.mark.gpu)]

DENSE = {"kind": "dense", "ff": 40}


def att(heads=4, kv=2, dim=6, vdim=10, scale=0.9, chunk=11, mlp=DENSE):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
                      "scale": scale, "mask": {"size": chunk}}}


def delta(heads=4, kv=2, dim=10, vdim=6, conv=4, mlp=DENSE):
    return {"type": "channel_delta", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}}


def lat(heads=3, dim=6, rot=4, vdim=8, rank=10, q_rank=14, scale=0.7, window=9,
        base=40.0, kv_from=None, mlp=DENSE):
    mx = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank,
          "q_rank": q_rank, "scale": scale, "mask": {"size": window},
          "rot": {"base": base, "dims": rot}}
    if kv_from is not None:
        mx["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": mx, "mlp": mlp}


def config(layers, width=32, vocab=50, eps=1e-5, streams=3):
    return {"architecture": "Lipulorn", "vocab": vocab, "width": width,
            "norm": {"eps": eps}, "streams": streams, "layers": layers}


# the borrowing layer is not next to its source, has other heads, sizes and a
# wider window; a second one borrows the same rows
MIXED = config([lat(), delta(), att(),
                lat(heads=2, dim=4, vdim=6, q_rank=9, window=15, scale=1.1, kv_from=0),
                delta(heads=2, kv=2, dim=16, vdim=16, conv=2, mlp=None),
                lat(heads=5, dim=2, vdim=4, q_rank=6, window=3, kv_from=0, mlp=None)])

# sizes in multiples of 16: bf16 prompt portions take the matrix-core kernels
SIXTEENS = config(
    [att(heads=8, kv=2, dim=32, vdim=16, scale=0.2, chunk=40),
     lat(heads=4, dim=16, rot=16, vdim=32, rank=48, q_rank=32, scale=0.2, window=24,
         base=1000.0),
     delta(heads=4, kv=2, dim=32, vdim=16, conv=3),
     lat(heads=4, dim=32, rot=16, vdim=16, rank=48, q_rank=24, scale=0.15, window=50,
         base=1000.0, kv_from=1)],
    width=64, vocab=80, streams=2)


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
    g = torch.Generator().manual_seed(5000 + seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def npy(t):
    return t.detach().double().cpu().numpy()


def check(got, want):
    err = (np.abs(npy(got) - want).max(-1) / want.std()).max()
    assert err < 2e-4, f"relative error {err:.3g}"


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


def one_run(n, at, slot, device):
    return sops.SeqMeta.build([(n, slot)],
                              torch.arange(at, at + n, dtype=torch.int32).to(device), device)


# ---------------------------------------------------------------------------
# mechanisms as functions: the product's ops against the oracle's
# ---------------------------------------------------------------------------
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,R,half", [(2, 9, 6), (4, 64, 8), (1, 5, 1)])
def test_latent_rows_and_query_rotation_by_halves(device, H, R, half):
    g = torch.Generator().manual_seed(8)
    T, bs = 21, 16
    x = torch.randn(T, R + 2 * half, generator=g)
    qfull = torch.randn(T, H, 7 + 2 * half, generator=g)
    w = torch.randn(R, generator=g)
    pos = torch.randint(0, 900, (T,), generator=g).int()
    f = torch.tensor([40.0 ** (-2.0 * i / (2 * half)) for i in range(half)])
    slots = torch.randperm(3 * bs, generator=g)[:T]
    slots[4] = -1
    dev = lambda t: t.to(device)
    wq = oracle.rotate_halves(npy(qfull[..., 7:]), pos.numpy(), 40.0)
    want = np.concatenate([oracle.rms_norm(npy(x[:, :R]), npy(w), 1e-4),
                           oracle.rotate_halves(npy(x[:, R:]), pos.numpy(), 40.0)], -1)
    for own in (True, False):  # a layer that borrows rows only rotates its queries
        cache = dev(torch.zeros(3, 1, bs, R + 2 * half))
        ql = dev(torch.zeros(T, H, R + 2 * half))
        sops.latent_rope_to_cache(dev(x) if own else None, dev(w) if own else None, 1e-4,
                                  dev(qfull)[..., 7:], ql[..., R:], dev(pos), dev(f), 1.0,
                                  cache if own else None, dev(slots), halves=True)
        flat = npy(cache).reshape(-1, R + 2 * half)
        for t in range(T):
            if own and slots[t] >= 0:
                assert np.abs(flat[slots[t]] - want[t]).max() < 2e-4
        assert np.count_nonzero(np.abs(flat).sum(-1)) == (T - 1 if own else 0)
        assert np.abs(npy(ql[..., R:]) - wq).max() < 2e-4
        assert np.abs(npy(ql[..., :R])).max() == 0


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D,Dv", [(4, 2, 6, 10), (6, 6, 64, 32), (5, 1, 1, 1), (3, 3, 100, 4),
                                      (2, 1, 600, 8)])
def test_unit_rms_heads_to_cache(device, H, G, D, Dv):
    g = torch.Generator().manual_seed(9)
    T, bs = 5, 16
    proj = torch.randn(T, (H + G) * D + G * Dv + 8, generator=g)
    q = proj[:, : H * D].unflatten(-1, (H, D))
    k = proj[:, H * D : (H + G) * D].unflatten(-1, (G, D))
    v = proj[:, (H + G) * D :][:, : G * Dv].unflatten(-1, (G, Dv))
    q0, k0, v0 = npy(q), npy(k), npy(v)
    p = proj.to(device)
    q = p[:, : H * D].unflatten(-1, (H, D))
    k = p[:, H * D : (H + G) * D].unflatten(-1, (G, D))
    v = p[:, (H + G) * D :][:, : G * Dv].unflatten(-1, (G, Dv))
    kc, vc = torch.zeros(2, G, bs, D).to(device), torch.zeros(2, G, bs, Dv).to(device)
    slots = torch.tensor([3, 31, -1, 0, 16])
    sops.headnorm_qk_to_cache(q, k, v, 1e-2, kc, vc, slots.to(device))
    assert np.abs(npy(q) - oracle.unit_rms(q0, 1e-2)).max() < 1e-5
    for t, s in enumerate(slots.tolist()):
        if s >= 0:
            assert np.abs(npy(kc)[s // bs, :, s % bs] - oracle.unit_rms(k0[t], 1e-2)).max() < 1e-5
            assert np.abs(npy(vc)[s // bs, :, s % bs] - v0[t]).max() < 1e-6
    assert np.count_nonzero(np.abs(npy(vc)).sum((1, 3))) == 4  # nothing else was written


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("S", [1, 2, 3, 4, 5, 8])
@pytest.mark.parametrize("C", [24, 37])
def test_stream_update_and_read(device, S, C):
    g = torch.Generator().manual_seed(S)
    X, y = torch.randn(6, S, C, generator=g), torch.randn(6, C, generator=g)
    mix, write = torch.randn(S, S, generator=g), torch.randn(S, generator=g)
    read, w = torch.randn(S, generator=g), torch.randn(C, generator=g)
    dev = lambda t: t.to(device)
    Xd = dev(X.clone())
    h = sops.hyper_mix_rmsnorm(Xd, dev(y), None, dev(mix), dev(write), dev(read), dev(w), 1e-3,
                               torch.float32)
    X1 = oracle.write_streams(npy(X), npy(y), npy(mix), npy(write))
    assert np.abs(npy(Xd) - X1).max() < 2e-5
    u = oracle.read_streams(X1, npy(read))
    assert np.abs(npy(h) - oracle.rms_norm(u, npy(w), 1e-3)).max() < 2e-5
    # reading alone leaves the streams as they are
    h = sops.hyper_mix_rmsnorm(Xd, None, None, None, None, dev(read), dev(w), 1e-3,
                               torch.float32)
    assert np.abs(npy(Xd) - X1).max() < 2e-5
    assert np.abs(npy(h) - oracle.rms_norm(u, npy(w), 1e-3)).max() < 2e-5


@pytest.mark.parametrize("device", DEVICES)
def test_streams_start_as_copies_of_the_embedding(device):
    table = torch.randn(7, 12).to(device)
    ids = torch.tensor([3, 0, 6, 3], dtype=torch.int32).to(device)
    X = npy(sops.embed_streams(ids, table, 3))
    assert X.shape == (4, 3, 12)
    assert (X == npy(table)[ids.cpu().numpy()][:, None]).all()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("taps,C", [(1, 9), (2, 16), (3, 40), (4, 8), (4, 9), (5, 16)])
def test_conv_silu_and_carried_tail(device, taps, C):
    """Runs around the number of tokens that one thread of the kernel walks,
    whole and in portions over a stale tail."""
    g = torch.Generator().manual_seed(7)
    T = 50
    x, w = torch.randn(T, C, generator=g), torch.randn(C, taps, generator=g)
    want = oracle.short_conv_silu(npy(x), npy(w))
    for cuts in ([T], [1, 2, 5, 42], [15, 1, 16, 1, 17], [17, 33], [1] * T):
        tails = torch.randn(2, taps - 1, C).to(device)
        got, at = [], 0
        for n in cuts:
            got.append(sops.causal_conv(x[at : at + n].to(device), w.to(device), tails,
                                        one_run(n, at, 1, device), False, act="silu"))
            at += n
        assert np.abs(npy(torch.cat(got)) - want).max() < 1e-5


@pytest.mark.parametrize("device", DEVICES)
def test_conv_unequal_batch(device):
    """A long run, single tokens that continue their tails, a run without a
    slot, all in one step."""
    g = torch.Generator().manual_seed(17)
    C, taps = 16, 4
    w = torch.randn(C, taps, generator=g)
    seqs = [torch.randn(n, C, generator=g) for n in (40, 9, 23, 5)]
    want = [oracle.short_conv_silu(npy(x), npy(w)) for x in seqs]
    tails = torch.randn(4, taps - 1, C).to(device)
    for i, n in ((1, 8), (2, 4)):
        sops.causal_conv(seqs[i][:n].to(device), w.to(device), tails, one_run(n, 0, i, device),
                         False, act="silu")
    parts = [(0, 0, 40), (1, 8, 9), (2, 4, 23), (3, 0, 5)]
    x = torch.cat([seqs[i][a:b] for i, a, b in parts]).to(device)
    pos = torch.cat([torch.arange(a, b) for _, a, b in parts]).int().to(device)
    meta = sops.SeqMeta.build([(b - a, -1 if i == 3 else i) for i, a, b in parts], pos, device)
    before = tails[3].clone()
    got = npy(sops.causal_conv(x, w.to(device), tails, meta, False, act="silu"))
    at = 0
    for i, a, b in parts:
        assert np.abs(got[at : at + b - a] - want[i][a:b]).max() < 1e-5
        at += b - a
    for i in range(3):
        assert np.abs(npy(tails[i]) - npy(seqs[i][-(taps - 1):])).max() < 1e-6
    assert (tails[3] == before).all()


def _delta_inputs(T, H, G, D, Dv, seed):
    g = torch.Generator().manual_seed(seed)
    q, k = torch.randn(T, G, D, generator=g), torch.randn(T, G, D, generator=g)
    v = torch.randn(T, H, Dv, generator=g)
    b, a = torch.randn(T, H, generator=g) * 2, torch.randn(T, H, D, generator=g) * 2
    a_log, dt = torch.randn(H, generator=g), torch.randn(H * D, generator=g)
    return q, k, v, b, a, a_log, dt


def _delta_want(q, k, v, b, a, a_log, dt):
    T, G, D = q.shape
    H = v.shape[1]
    qn, kn = oracle.unit_vectors(npy(q)) * D ** -0.5, oracle.unit_vectors(npy(k))
    beta = oracle.sigmoid(npy(b))
    dec = oracle.channel_decay(npy(a).reshape(T, -1), npy(a_log), npy(dt))
    return np.stack([oracle.delta_recurrence(qn[:, h // (H // G)], kn[:, h // (H // G)],
                                             npy(v)[:, h], beta[:, h], dec[:, h])
                     for h in range(H)], axis=1)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D,Dv", [(4, 2, 10, 6), (2, 2, 16, 16), (3, 1, 32, 20),
                                      (1, 1, 3, 70), (2, 1, 48, 33)])
def test_channel_decay_scan_and_carried_state(device, H, G, D, Dv):
    """One run in one call, against the same tokens cut into calls that carry
    the state in a slot which held another sequence before."""
    T = 23
    ins = _delta_inputs(T, H, G, D, Dv, 5)
    want = _delta_want(*ins)
    dev = lambda t: t.to(device)
    state = torch.randn(3, H, D, Dv).to(device)  # stale contents of the slots
    for cuts in ([T], [9, 1, 13], [1] * T):
        got, at = [], 0
        for n in cuts:
            got.append(sops.gated_delta_scan(
                *(dev(t[at : at + n]) for t in ins[:5]), dev(ins[5]), dev(ins[6]), state,
                one_run(n, at, 1, device)))
            at += n
        assert np.abs(npy(torch.cat(got)) - want).max() < 2e-5


@pytest.mark.parametrize("device", DEVICES)
def test_channel_decay_scan_long_run_and_unequal_batch(device):
    """A 600-token run (cut into parallel segments on the GPU) beside a short
    one and a single token that continues a stored state."""
    H, G, D, Dv = 2, 1, 16, 20
    ins = _delta_inputs(600, H, G, D, Dv, 6)
    short = _delta_inputs(37, H, G, D, Dv, 7)[:5] + ins[5:]
    want, want_s = _delta_want(*ins), _delta_want(*short)
    dev = lambda t: t.to(device)
    state = torch.zeros(4, H, D, Dv).to(device)
    sops.gated_delta_scan(*(dev(t[:36]) for t in short[:5]), dev(ins[5]), dev(ins[6]), state,
                          one_run(36, 0, 2, device))
    pos = torch.cat([torch.arange(600), torch.arange(37), torch.tensor([36])]).int().to(device)
    meta = sops.SeqMeta.build([(600, 0), (37, 3), (1, 2)], pos, device)
    cat = [torch.cat([ins[j], short[j], short[j][36:37]]) for j in range(5)]
    got = npy(sops.gated_delta_scan(*(dev(t) for t in cat), dev(ins[5]), dev(ins[6]), state,
                                    meta))
    assert np.abs(got[:600] - want).max() < 5e-5
    assert np.abs(got[600:637] - want_s).max() < 5e-5
    assert np.abs(got[637] - want_s[36]).max() < 5e-5


@pytest.mark.parametrize("device", DEVICES)
def test_decay_belongs_to_its_own_channel(device):
    """Two keys along two channels of one head, written once; afterwards one
    channel is kept and the other forgotten, and heads do not mix."""
    H, D, Dv, T = 2, 16, 16, 4
    k = torch.zeros(T, 1, D)
    k[0, 0, 2], k[1, 0, 5], k[2:, 0, 9] = 3.0, 3.0, 3.0
    q = torch.zeros(T, 1, D)
    q[:, 0, 2] = 1.0
    q[3, 0, 2], q[3, 0, 5] = 0.0, 1.0
    v = torch.zeros(T, H, Dv)
    v[0, :, 1], v[1, :, 3] = 4.0, 6.0
    b = torch.full((T, H), 30.0)
    a = torch.full((T, H, D), -40.0)  # softplus -> 0: decay 1
    a[2, 0, 2] = 40.0                 # head 0 forgets channel 2 at token 2
    a[3, 1, 5] = 40.0                 # head 1 forgets channel 5 at token 3
    state = torch.zeros(1, H, D, Dv).to(device)
    o = npy(sops.gated_delta_scan(*(t.to(device) for t in (q, k, v, b, a)),
                                  torch.zeros(H).to(device), torch.zeros(H * D).to(device),
                                  state, one_run(T, 0, 0, device))) * D ** 0.5
    assert abs(o[1, 0, 1] - 4) < 1e-4 and abs(o[1, 1, 1] - 4) < 1e-4
    assert abs(o[2, 0, 1]) < 1e-4 and abs(o[2, 1, 1] - 4) < 1e-4
    assert abs(o[3, 0, 3] - 6) < 1e-4 and abs(o[3, 1, 3]) < 1e-4


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("D", [16, 24])
def test_decays_near_one_keep_their_accuracy(device, D):
    """Two hundred steps without writes whose decays differ from one by 1e-7 to
    1: the remaining state gives each channel's product of decays. A decay's
    logarithm has to be right relative to itself, or slow channels drift."""
    T = 200
    pre = torch.linspace(-17.0, 3.0, D).view(1, 1, D).expand(T, 1, D).contiguous()
    pre[:, :, -1] = 25.0  # beyond where softplus is the identity
    k = torch.zeros(T, 1, D)
    v = torch.zeros(T, 1, 2)
    state = torch.ones(1, 1, D, 2).to(device)
    a_log = torch.tensor([-3.0])
    meta = sops.SeqMeta.build([(T, 0)], torch.arange(5, 5 + T, dtype=torch.int32).to(device),
                              device)
    sops.gated_delta_scan(*(t.to(device) for t in (k, k, v, torch.zeros(T, 1), pre)),
                          a_log.to(device), torch.zeros(D).to(device), state, meta)
    log = -np.exp(-3.0) * T * oracle.softplus(npy(pre[0, 0]))
    got = npy(state)[0, 0, :, 0]
    assert np.abs(got - np.exp(log)).max() < 3e-5
    slow = np.abs(log) < 0.05
    assert slow.sum() >= 4  # what is left of these channels is 1 - (a small number)
    assert np.abs((1 - got[slow]) - -np.expm1(log[slow])).max() < 2e-5


# ---------------------------------------------------------------------------
# every mechanism alone, in the engine
# ---------------------------------------------------------------------------
SINGLE = {
    "chunk_attention_no_ff": config([att(mlp=None)]),
    "delta_no_ff": config([delta(mlp=None)]),
    "latent_no_ff": config([lat(mlp=None)]),
    "latent_borrowed_no_ff": config([lat(mlp=None), lat(kv_from=0, window=5, mlp=None)]),
    "attention_with_ff": config([att()]),
    "delta_with_ff": config([delta()]),
    "one_stream": config([lat(), delta()], streams=1),
    "heads_own_their_keys": config([att(heads=3, kv=3), delta(heads=3, kv=3)]),
    "one_key_head": config([att(heads=5, kv=1, dim=3), delta(heads=4, kv=1)]),
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", sorted(SINGLE))
def test_single_mechanism(tmp_path, device, name):
    cfg = SINGLE[name]
    d, W = model_dir(tmp_path, cfg, seed=3)
    toks = tokens(37, cfg["vocab"], 1)
    want = oracle.forward(cfg, W, toks)
    eng = engine(d, device)
    check(replay(eng, "a", toks, [len(toks)]), want)
    check(replay(eng, "b", toks, [20, 2, 1]), want)


@pytest.mark.parametrize("device", DEVICES)
def test_streams_match_after_every_layer(tmp_path, device):
    d, W = model_dir(tmp_path, MIXED, seed=4)
    toks = tokens(29, MIXED["vocab"], 2)
    layers = []
    oracle.forward(MIXED, W, toks, capture=layers)
    eng = engine(d, device)
    eng.runner.model.capture_layers = []
    replay(eng, "a", toks, [len(toks)])
    got = torch.stack(eng.runner.model.capture_layers)[:, : len(toks)]
    assert got.shape[0] == len(layers) == 6
    for i, want in enumerate(layers):
        check(got[i], want)


# ---------------------------------------------------------------------------
# prompt vs decoding, portions, first tokens
# ---------------------------------------------------------------------------
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cuts", [[1], [2], [3, 2, 5], [7, 1, 1, 4, 1], [16, 1], [11, 13]])
def test_portions_and_token_by_token(tmp_path, device, cuts):
    d, W = model_dir(tmp_path, MIXED, seed=5)
    toks = tokens(45, MIXED["vocab"], 3)
    check(replay(engine(d, device), "a", toks, cuts), oracle.forward(MIXED, W, toks))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("n", [1, 2, 3])
def test_first_tokens(tmp_path, device, n):
    d, W = model_dir(tmp_path, MIXED, seed=6)
    toks = tokens(n, MIXED["vocab"], 4)
    want = oracle.forward(MIXED, W, toks)
    check(replay(engine(d, device), "a", toks, [n]), want)
    check(replay(engine(d, device), "b", toks, [1]), want)


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding(tmp_path, device):
    d, W = model_dir(tmp_path, MIXED, seed=7)
    toks = tokens(130, MIXED["vocab"], 5)
    check(replay(engine(d, device), "a", toks, [9, 1]), oracle.forward(MIXED, W, toks))


@pytest.mark.parametrize("device", DEVICES)
def test_long_prompt(tmp_path, device):
    """Longer than the run length from which the delta scan works in segments
    (GPU), in one step and in portions."""
    cfg = config([delta(heads=2, kv=1, dim=16, vdim=12), lat(window=130), att(chunk=70)])
    d, W = model_dir(tmp_path, cfg, seed=8)
    toks = tokens(310, cfg["vocab"], 6)
    want = oracle.forward(cfg, W, toks)
    check(replay(engine(d, device), "a", toks, [len(toks)]), want)
    check(replay(engine(d, device), "b", toks, [280, 2, 1]), want)


@pytest.mark.parametrize("device", GPU)
@pytest.mark.parametrize("name", ["mixed", "sixteens"])
def test_bfloat16_serving_precision(tmp_path, device, name):
    """The widths are tiny, so roundings do not average out: with the odd sizes
    the reference ops on the CPU put single positions at 0.7 in bf16. Most
    positions stay close."""
    cfg = {"mixed": MIXED, "sixteens": SIXTEENS}[name]
    d, W = model_dir(tmp_path, cfg, seed=9)
    toks = tokens(90, cfg["vocab"], 7)
    want = oracle.forward(cfg, W, toks)
    for rid, cuts in (("a", [len(toks)]), ("b", [33, 2, 1])):
        got = npy(replay(engine(d, device, "bfloat16"), rid, toks, cuts))
        err = np.abs(got - want).max(-1) / want.std()
        assert np.median(err) < 0.1 and np.quantile(err, 0.9) < 0.2
        assert name == "mixed" or err.max() < 0.15
    check(replay(engine(d, device), "c", toks, [33, 2, 1]), want)


# ---------------------------------------------------------------------------
# batches, reuse of blocks and slots
# ---------------------------------------------------------------------------
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


# ---------------------------------------------------------------------------
# edges of windows and chunks: one score made to stand out
# ---------------------------------------------------------------------------
def _planted(device, q_pos, key_pos, window=0, chunk=0, block=16, decode=False,
             dtype=torch.float32, H=4, G=2, D=8, Dv=8, tied=0, gated=True):
    """Only key_pos has a key aligned with the queries, with values of 7.
    tied: one row per token whose first Dv columns are the value. Returns (got,
    want, gates) for the query at q_pos."""
    T = q_pos + 1
    k, v = torch.zeros(T, G, D), torch.zeros(T, G, Dv)
    k[key_pos, :, 0] = 48.0
    v[key_pos] = 7.0
    if tied:
        v[:, :, 0] = k[:, :, 0]
        k[:, :, :Dv] = v
    q = torch.zeros(T, H, D)
    q[:, :, 0] = 1.0
    gate = torch.linspace(-1.0, 2.0, T * (H + 3)).view(T, H + 3)[:, 1 : H + 1]
    seen = (oracle.window_mask(T, window) if window else oracle.chunk_mask(T, chunk))
    want = []
    for h in range(H):
        g = h // (H // G)
        a = oracle.masked_softmax(npy(q[:, h]) @ npy(k[:, g]).T, seen)
        want.append((a @ npy(v[:, g]))[q_pos])
    gates = oracle.sigmoid(npy(gate.to(dtype).float()))[q_pos] if gated else np.ones(H)
    want = np.stack(want) * gates[:, None]
    nblk = (T + block - 1) // block
    perm = torch.randperm(nblk + 3, generator=torch.Generator().manual_seed(T)).tolist()
    table = torch.tensor([perm[:nblk]], dtype=torch.int32)
    kc, vc = torch.zeros(nblk + 3, G, block, D), torch.zeros(nblk + 3, G, block, Dv)
    tp = torch.arange(T)
    kc[table[0][tp // block].long(), :, tp % block] = k
    vc[table[0][tp // block].long(), :, tp % block] = v
    lo = q_pos if decode else max(0, q_pos - 20)
    positions = torch.arange(lo, q_pos + 1, dtype=torch.int32)
    meta = sops.SeqMeta.build([(q_pos + 1 - lo, 0)], positions.to(device), device,
                              block_tables=table.to(device))
    out = torch.zeros(q_pos + 1 - lo, H, Dv, device=device, dtype=dtype)
    kc, vc = kc.to(device, dtype), vc.to(device, dtype)
    sops.masked_paged_attention(q[lo:].to(device, dtype).contiguous(), kc,
                                kc[..., :Dv] if tied else vc, meta, 1.0, out, window=window,
                                chunk=chunk,
                                head_gate=gate[lo:].to(device, dtype) if gated else None)
    return npy(out[-1].float()), want, gates


# (position, window or 0, chunk or 0): the farthest visible token and the one behind it
EDGES = [(40, 9, 0), (47, 16, 0), (48, 17, 0), (300, 128, 0), (300, 33, 0), (31, 1, 0),
         (21, 0, 11), (22, 0, 11), (32, 0, 11), (48, 0, 16), (63, 0, 16), (299, 0, 100),
         (300, 0, 100), (5, 0, 1), (700, 0, 512)]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("pos,window,chunk", EDGES)
def test_planted_key_at_the_edge(device, decode, pos, window, chunk):
    first = pos - window + 1 if window else pos // chunk * chunk
    got, want, gates = _planted(device, pos, first, window, chunk, decode=decode)
    assert np.abs(want[:, 1] - 7.0 * gates).max() < 1e-6  # the planted key has all the weight
    assert np.abs(got - want).max() < 1e-4
    if first > 0:
        got, want, _ = _planted(device, pos, first - 1, window, chunk, decode=decode)
        assert np.abs(want).max() == 0 and np.abs(got).max() < 1e-6


@pytest.mark.parametrize("device", GPU)
@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("pos,window,chunk", EDGES)
@pytest.mark.parametrize("sizes", [
    dict(H=4, G=2, D=16, Dv=32), dict(H=8, G=2, D=64, Dv=64), dict(H=4, G=1, D=48, Dv=80),
    dict(H=8, G=1, D=64, Dv=48, tied=1), dict(H=16, G=1, D=192, Dv=128, tied=1)],
    ids=lambda s: "-".join(str(v) for v in s.values()))
def test_planted_key_at_the_edge_matrix_core_kernels(device, decode, pos, window, chunk, sizes):
    first = pos - window + 1 if window else pos // chunk * chunk
    got, want, _ = _planted(device, pos, first, window, chunk, decode=decode,
                            dtype=torch.bfloat16, **sizes)
    assert np.abs(got - want).max() < 0.25 and np.abs(want).max() > 1
    if first > 0:
        got, want, _ = _planted(device, pos, first - 1, window, chunk, decode=decode,
                                dtype=torch.bfloat16, gated=False, **sizes)
        assert np.abs(got).max() < 1e-6


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind", ["window", "chunk", "borrowed"])
def test_logits_ignore_the_token_outside_and_notice_the_one_inside(tmp_path, device, kind):
    """One attention layer: changing the token just outside the last position's
    window or chunk leaves its logits alone, changing the one just inside
    moves them as the oracle says; prompt, portions across the edge, decoding."""
    layers = {"window": [lat(window=20, scale=0.1, mlp=None)],
              "chunk": [att(chunk=20, scale=0.1, mlp=None)],
              # the borrowing layer's own window is the wider one; one layer's
              # reach behind the other's is what the streams carry
              "borrowed": [lat(window=1, mlp=None),
                           lat(window=20, scale=0.1, kv_from=0, mlp=None)]}[kind]
    cfg = config(layers)
    d, W = model_dir(tmp_path, cfg, seed=13)
    n = 20 + 35 if kind == "chunk" else 50  # chunk: position 54, chunk 40..59
    first = 40 if kind == "chunk" else n - 20
    base = tokens(n, cfg["vocab"], 8)

    def changed(i):
        t = list(base)
        t[i] = (t[i] + 1) % cfg["vocab"]
        return t

    eng = engine(d, device)
    want = oracle.forward(cfg, W, base)[-1]
    for c, cuts in enumerate([[n], [first + 3, 2, n], [n - 6, 1], [first - 1, 2, 3, n]]):
        r = [npy(replay(eng, "%d%d" % (c, i), t, cuts)[-1])
             for i, t in enumerate([base, changed(first - 1), changed(first)])]
        assert np.abs(r[0] - want).max() / want.std() < 2e-4
        assert np.abs(r[1] - r[0]).max() / want.std() < 1e-5
        moved = oracle.forward(cfg, W, changed(first))[-1] - want
        assert np.abs(moved).max() > 1e-3 * want.std()
        assert np.abs((r[2] - r[0]) - moved).max() / want.std() < 2e-4


@pytest.mark.parametrize("device", DEVICES)
def test_far_token_reaches_logits_through_the_state_alone(tmp_path, device):
    cfg = config([delta(heads=2, kv=1, dim=64, vdim=8, mlp=None)])
    W = oracle.random_weights(cfg, 14)
    W["l0.mix.A_log"] = torch.full_like(W["l0.mix.A_log"], -6.0)  # slow decay
    d, W = model_dir(tmp_path, cfg, seed=14, W=W)
    a = tokens(300, cfg["vocab"], 31)
    b = list(a)
    b[2] = (a[2] + 1) % cfg["vocab"]
    eng = engine(d, device)
    ga = npy(replay(eng, "a", a, [250, 3, 1])[-1])
    gb = npy(replay(eng, "b", b, [250, 3, 1])[-1])
    wa, wb = oracle.forward(cfg, W, a)[-1], oracle.forward(cfg, W, b)[-1]
    assert np.abs(wa - wb).max() > 1e-4 * wa.std()
    assert np.abs((ga - gb) - (wa - wb)).max() / wa.std() < 2e-4


# ---------------------------------------------------------------------------
# other sizes and orders
# ---------------------------------------------------------------------------
OTHER = {
    "delta_first": config(
        [delta(heads=6, kv=3, dim=4, vdim=2, conv=3), lat(heads=5, dim=2, rot=6, vdim=2, rank=12),
         att(heads=6, kv=3, dim=2, vdim=20, chunk=7)], width=24, vocab=33, streams=5),
    "one_of_everything": config(
        [att(heads=1, kv=1, dim=1, vdim=1, chunk=1), lat(heads=1, dim=1, rot=2, vdim=1, rank=1,
                                                        q_rank=1, window=1),
         delta(heads=1, kv=1, dim=1, vdim=1, conv=2)], width=16, streams=1),
    "no_convolution_history": config([delta(conv=1), delta(conv=6, heads=2, kv=1)], eps=1e-3),
    "wide_rotation_small_latent": config(
        [lat(heads=2, dim=2, rot=20, vdim=6, rank=3, base=7.0, scale=1.3, window=100),
         delta(), lat(heads=8, dim=4, rot=20, vdim=2, rank=3, base=7.0, q_rank=30, kv_from=0)],
        width=16, eps=1e-3, streams=4),
    "masks_larger_than_the_prompt": config([lat(window=500), att(chunk=500)], width=40, vocab=70),
    "aligned_sizes": SIXTEENS,
    "key_size_of_forty_eight": config([delta(heads=2, kv=1, dim=48, vdim=40),
                                       att(heads=6, kv=2, dim=16, vdim=48, chunk=16)],
                                      width=48, streams=2),
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", sorted(OTHER))
def test_other_sizes(tmp_path, device, name):
    cfg = OTHER[name]
    d, W = model_dir(tmp_path, cfg, seed=15)
    toks = tokens(40, cfg["vocab"], 32)
    check(replay(engine(d, device), "a", toks, [13, 2, 1]), oracle.forward(cfg, W, toks))


def test_bottleneck_sizes_come_from_the_checkpoint(tmp_path):
    cfg = config([delta()])
    for i, rank in enumerate((1, 8, 13)):
        d, W = model_dir(tmp_path, cfg, seed=60 + i,
                         W=oracle.random_weights(cfg, 60 + i, low_rank=rank))
        eng = engine(d, "cpu")
        m = eng.runner.model.layers[0].mixer
        assert (m.decay_rank, m.gate_rank) == (rank, rank + 2)
        toks = tokens(12, cfg["vocab"], 33)
        check(replay(eng, "a", toks, [12]), oracle.forward(cfg, W, toks))


def test_loader_and_config_errors(tmp_path):
    cfg = config([lat(), lat(kv_from=0)])
    W = oracle.random_weights(cfg, 16)
    W["l1.mix.dkv"] = torch.zeros(14, 32).bfloat16()  # a borrowing layer has none
    with pytest.raises(ValueError, match="not consumed"):
        engine(model_dir(tmp_path, cfg, seed=16, W=W)[0], "cpu")
    W = oracle.random_weights(cfg, 17)
    del W["l1.hc2.mix"]
    with pytest.raises(ValueError, match="hc2.mix"):
        engine(model_dir(tmp_path, cfg, seed=17, W=W)[0], "cpu")
    bad = {
        "earlier": [lat(kv_from=0)],
        "caches no latent": [delta(), lat(kv_from=0)],
        "kv_rank differs": [lat(), lat(rank=11, kv_from=0)],
        "rot differs": [lat(), lat(base=41.0, kv_from=0)],
        "at least one token": [att(chunk=0)],
        "unknown mixer": [dict(att(), type="mingru")],
        "unknown feed-forward": [att(mlp={"kind": "moe"})],
    }
    for i, (msg, layers) in enumerate(bad.items()):
        good = config([lat()])
        with pytest.raises(ValueError, match=msg):
            engine(model_dir(tmp_path, config(layers), seed=70 + i,
                             W=oracle.random_weights(good, 1))[0], "cpu")


def test_what_is_kept_per_token_and_sequence(tmp_path):
    d, _ = model_dir(tmp_path, MIXED, seed=19)
    r = engine(d, "cpu").runner
    kv = [None if c is None else (c[0].shape[1], c[0].shape[-1], c[1].shape[-1])
          for c in r.kv_caches]
    # latent + rotated key part; nothing where a layer borrows or keeps a state
    assert kv == [(1, 14, 0), None, (2, 6, 10), None, None, None]
    m = r.model
    assert m.kv_caches[3] is m.kv_caches[0] and m.kv_caches[5] is m.kv_caches[0]
    assert [sorted(s) for s in r.states] == [[], ["conv", "s"], [], [], ["conv", "s"], []]
    assert r.states[1]["s"].shape[1:] == (4, 10, 6)
    assert r.states[1]["conv"].shape[1:] == (3, 2 * 20 + 24)


# ---------------------------------------------------------------------------
# generation through the engine's own entry point and scheduler
# ---------------------------------------------------------------------------
def _generate(eng, prompts, max_tokens, arrive_every=0):
    pending = list(prompts.items())
    params = SamplingParams(max_tokens=max_tokens, ignore_eos=True)
    if not arrive_every:
        for rid, t in pending:
            eng.add_request(t, params, request_id=rid)
        pending = []
    done, steps = {}, 0
    while (pending or eng.has_work()) and steps < 600:
        if pending and steps % arrive_every == 0:
            rid, t = pending.pop(0)
            eng.add_request(t, params, request_id=rid)
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


def test_preemption_and_abort_keep_cache_and_state_consistent(tmp_path):
    d, W = model_dir(tmp_path, MIXED, seed=21)
    eng = LLMEngine(EngineConfig(
        model=d, device="cpu", dtype="float32", num_gpu_blocks=6, max_num_seqs=3,
        max_model_len=128, max_num_batched_tokens=64))  # tight pool: preemption
    prompts = {"q%d" % i: tokens(30, MIXED["vocab"], 70 + i) for i in range(3)}
    for rid, t in prompts.items():
        eng.add_request(t, SamplingParams(max_tokens=20, ignore_eos=True), request_id=rid)
    done, steps = {}, 0
    while eng.has_work() and steps < 600:
        if steps == 3:
            eng.abort_request("q1")
        for o in eng.step():
            if o.finished:
                done[o.request_id] = list(o.output_token_ids)
        steps += 1
    _assert_greedy(MIXED, W, {r: prompts[r] for r in ("q0", "q2")},
                   {r: done[r] for r in ("q0", "q2")}, 1e-3)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_decode_graph_replays_match_oracle(tmp_path, dtype):
    """Pure-decode steps replay a captured graph; prompt portions of later
    arrivals run eagerly between replays. Every generated token is checked."""
    cfg = MIXED if dtype == "float32" else SIXTEENS
    d, W = model_dir(tmp_path, cfg, seed=22)
    eng = LLMEngine(EngineConfig(
        model=d, device="cuda", dtype=dtype, num_gpu_blocks=64, max_num_seqs=6,
        max_model_len=512, max_num_batched_tokens=64, enable_graphs=True))
    prompts = {"g%d" % i: tokens(n, cfg["vocab"], 90 + i)
               for i, n in enumerate([9, 33, 4, 70, 18, 2, 25])}
    done = _generate(eng, prompts, 24, arrive_every=5)
    assert eng.runner._graphs, "no decode graph was captured"
    _assert_greedy(cfg, W, prompts, done, 1e-3 if dtype == "float32" else 0.25)


def test_preset_builds_and_generates():
    eng = LLMEngine(EngineConfig(model="lipulorn-tiny", device="cpu", dtype="float32",
                                 num_gpu_blocks=16, max_num_seqs=2, max_model_len=128))
    eng.add_request(tokens(9, 512, 1), SamplingParams(max_tokens=4, ignore_eos=True),
                    request_id="r")
    out = []
    while eng.has_work():
        out += [o for o in eng.step() if o.finished]
    assert len(out) == 1 and len(out[0].output_token_ids) == 4


# ---------------------------------------------------------------------------
# kernels one by one against the reference ops (GPU)
# ---------------------------------------------------------------------------
def _close(got, want, dtype):
    tol = 2e-5 if dtype == torch.float32 else 2e-2
    scale = max(1.0, float(want.abs().max()))
    assert float((got.float().cpu() - want.float()).abs().max()) <= tol * scale


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("S,C", [(1, 256), (2, 1000), (3, 512), (4, 2048), (4, 4100), (4, 38),
                                 (2, 9000)])
def test_kernel_streams(dtype, S, C):
    g = torch.Generator().manual_seed(C)
    T = 5
    X = torch.randn(T, S, C, generator=g)
    y = torch.randn(T, C, generator=g)
    gate = torch.randn(T, C + 4, generator=g).to(dtype)[:, 4:]
    mix, wr, rd = (torch.randn(*s, generator=g) for s in ((S, S), (S,), (S,)))
    w = torch.randn(C, generator=g)
    for yy in (y.to(dtype), y):
        for gg in (None, gate):
            X_ref, X_gpu = X.clone(), X.clone().cuda()
            want = sops.hyper_mix_rmsnorm(X_ref, yy, gg, mix, wr, rd, w, 1e-5, dtype)
            got = sops.hyper_mix_rmsnorm(X_gpu, yy.cuda(), None if gg is None else gg.cuda(),
                                         mix.cuda(), wr.cuda(), rd.cuda(), w.cuda(), 1e-5, dtype)
            _close(X_gpu, X_ref, torch.float32)
            _close(got, want, dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("groups,gs", [(3, 16), (2, 128), (4, 100), (1, 256), (2, 300), (5, 6)])
@pytest.mark.parametrize("act", ["none", "sigmoid", "silu"])
def test_kernel_gated_norm(dtype, groups, gs, act):
    g = torch.Generator().manual_seed(gs)
    T, C = 7, groups * gs
    o = torch.randn(T, C, generator=g)
    w = torch.randn(C, generator=g)
    gate = torch.randn(T, C + 8, generator=g).to(dtype)
    res = []
    for dev in ("cpu", "cuda"):
        out = torch.zeros(T, C + 4, dtype=dtype, device=dev)
        sops.gated_rmsnorm(o.to(dev), w.to(dev), gate.to(dev)[:, 8:], groups, act, 1e-4,
                           out[:, 4:], 0.7)
        res.append(out)
    _close(res[1], res[0], dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D,Dv", [(4, 2, 32, 16), (2, 1, 128, 40), (3, 3, 10, 6),
                                      (8, 4, 64, 64), (2, 1, 48, 24), (1, 1, 80, 100),
                                      (2, 2, 16, 300), (1, 1, 200, 260), (2, 1, 112, 33),
                                      (2, 1, 96, 128)])
def test_kernel_channel_delta_scan(dtype, H, G, D, Dv):
    """Register-state and LDS-state kernels, plain and segment-parallel runs,
    inputs as strided column views of wider rows, against the reference."""
    lens = [(600, 0), (1, 2), (70, 1), (3, -1)]
    T = sum(n for n, _ in lens)
    g = torch.Generator().manual_seed(D)
    nqk, nv = G * D, H * Dv
    proj = torch.randn(T, 2 * nqk + nv + H, generator=g).to(dtype)
    pre = (torch.randn(T, H * D + 8, generator=g) * 2).to(dtype)
    a_log, dt = torch.randn(H, generator=g), torch.randn(H * D, generator=g)
    pos = torch.cat([torch.arange(600), torch.tensor([41]), torch.arange(5, 75),
                     torch.arange(3)]).int()
    state0 = torch.randn(3, H, D, Dv, generator=g) * 0.1
    res = []
    for dev in ("cpu", "cuda"):
        p = proj.to(dev)
        st = state0.clone().to(dev)
        meta = sops.SeqMeta.build(lens, pos.to(dev), dev)
        o = sops.gated_delta_scan(
            p[:, :nqk].unflatten(-1, (G, D)), p[:, nqk : 2 * nqk].unflatten(-1, (G, D)),
            p[:, 2 * nqk : 2 * nqk + nv].unflatten(-1, (H, Dv)), p[:, 2 * nqk + nv :],
            pre.to(dev)[:, : H * D].unflatten(-1, (H, D)), a_log.to(dev), dt.to(dev), st, meta)
        res.append((o.cpu(), st.cpu()))
    assert float((res[1][0] - res[0][0]).abs().max()) < 1e-4
    assert float((res[1][1] - res[0][1]).abs().max()) < 1e-4


@pytest.mark.gpu
@pytest.mark.parametrize("n", [127, 128, 129, 256, 257, 513])
def test_kernel_scan_at_segment_borders(n):
    ins = _delta_inputs(n, 2, 1, 16, 8, n)
    state = torch.zeros(1, 2, 16, 8).cuda()
    got = sops.gated_delta_scan(*(t.cuda() for t in ins), state, one_run(n, 0, 0, "cuda"))
    assert np.abs(npy(got) - _delta_want(*ins)).max() < 5e-5


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D,Dv,mask", [
    (4, 2, 6, 10, dict(chunk=17)), (8, 2, 128, 128, dict(chunk=64)),
    (16, 4, 64, 64, dict(chunk=50)), (8, 4, 48, 80, dict(chunk=40)),
    (16, 1, 192, 128, dict(window=48)), (8, 1, 160, 128, dict(window=30)),
    (16, 4, 128, 128, dict()), (3, 3, 16, 16, dict(window=7))])
def test_kernel_gated_masked_attention(dtype, H, G, D, Dv, mask):
    """Prompt portions and split decoding with a gate per head (a strided slice
    of wider rows), for caches of separate and of tied rows."""
    g = torch.Generator().manual_seed(H + D)
    bs, nblk = 16, 24
    lens = [(40, 300), (1, 277), (9, 9), (1, 1)]  # (run length, sequence length)
    tied = G == 1
    kc = (torch.randn(nblk * 4, G, bs, D, generator=g) * 0.5).to(dtype)
    vc = (torch.randn(nblk * 4, G, bs, Dv, generator=g) * 0.5).to(dtype)
    tables = torch.stack([torch.randperm(nblk * 4, generator=g)[:nblk] for _ in lens]).int()
    pos = torch.cat([torch.arange(L - n, L) for n, L in lens]).int()
    T = int(pos.numel())
    q = (torch.randn(T, H, D, generator=g) * 0.5).to(dtype)
    gate = torch.randn(T, H + 5, generator=g).to(dtype)
    for decode_only in (False, True):
        if decode_only:
            runs, p, tb, n = [(1, 0)] * 3, torch.tensor([299, 276, 0]).int(), tables[:3], 3
        else:
            runs, p, tb, n = [(n, 0) for n, _ in lens], pos, tables, T
        outs = []
        for dev in ("cpu", "cuda"):
            meta = sops.SeqMeta.build(runs, p.to(dev), dev, block_tables=tb.to(dev))
            k, v = kc.to(dev), vc.to(dev)
            out = torch.zeros(n, H, Dv, dtype=dtype, device=dev)
            sops.masked_paged_attention(q[:n].to(dev), k, k[..., :Dv] if tied else v, meta,
                                        D ** -0.5, out, head_gate=gate[:n].to(dev)[:, 5:],
                                        out_scale=0.8, **mask)
            outs.append(out)
        _close(outs[1], outs[0].cpu(), dtype)
