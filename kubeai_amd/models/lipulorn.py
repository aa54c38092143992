"""Lipulorn: a decoder whose config lists its layers, built around several
residual streams (hyper-connections). Every sublayer q of a layer reads a
learned combination of the streams and writes back into all of them:

    u = sum_s in_q[s] x_s;  y = sublayer(rmsnorm(u) * w_q)
    x_t <- sum_s mix_q[s, t] x_s + out_q[t] * y            (all t at once)

The streams start as copies of the embedding and are summed at the end.
Mixers: the gated delta rule with a decay per key channel; latent attention
over a sliding window, with a query latent and a rotated key part, whose cached
rows another layer may have made; position-aligned chunk attention with unit
RMS queries and keys and a gate per head (kubeai_amd.models.mixers). The
feed-forward is a dense silu-gated layer with biases.

Same execution model as the other layer-list decoders: one token-packed
forward per engine step, GEMMs through the BLAS library in the serving dtype,
everything else in the gfx950 kernels of kubeai_amd.ops.seq. The streams are
fp32; a sublayer's write into the streams, the read for the next sublayer
and its norm are one kernel.
"""
from __future__ import annotations

import torch
import torch.nn as nn
import torch.nn.functional as F

from kubeai_amd.engine.batch import ForwardBatch
from kubeai_amd.ops import seq as sops
from .config import HybridLayerSpec, ModelArchConfig
from .mixers import (
    GatedDeltaMixer,
    HeadGatedAttention,
    HyperConnection,
    LatentAttention,
    SiluGatedMLP,
    _f32,
)


def mask_size(mixer: dict) -> int:
    size = int(mixer["mask"]["size"])
    if size < 1:
        raise ValueError("a window or chunk holds at least one token")
    return size


def build_mixer(spec: HybridLayerSpec, width: int, eps: float) -> nn.Module:
    m = spec.mixer
    if spec.type == "attention":
        return HeadGatedAttention(
            width, heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]),
            vdim=int(m["vdim"]), scale=m["scale"], chunk=mask_size(m), eps=eps,
        )
    if spec.type == "latent_attention":
        rot_dim = int(m["rot_dim"])
        if int(m["rot"]["dims"]) != rot_dim:
            raise ValueError("the rotated key part is rotated as a whole")
        return LatentAttention(
            width, heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
            kv_rank=int(m["kv_rank"]), scale=m["scale"],
            own_latent=m.get("kv_from") is None, eps=eps, q_rank=int(m["q_rank"]),
            rot_dim=rot_dim, rot_base=float(m["rot"]["base"]), rot_halves=True,
            gate=None, window=mask_size(m),
        )
    if spec.type == "channel_delta":
        low = max(8, width // 16)  # a checkpoint's tensors give the size
        return GatedDeltaMixer(
            width, heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]),
            vdim=int(m["vdim"]), conv_taps=int(m["conv"]), eps=eps, channel_decay=True,
            decay_rank=low, gate_rank=low, gate_act="sigmoid",
        )
    raise ValueError(f"unknown mixer type {spec.type!r}")


def build_mlp(mlp: dict | None, width: int):
    if mlp is None:
        return None
    if mlp.get("kind") == "dense":
        return SiluGatedMLP(width, int(mlp["ff"]), bias=True)
    raise ValueError(f"unknown feed-forward kind {mlp.get('kind')!r}")


class LipulornLayer(nn.Module):
    def __init__(self, spec: HybridLayerSpec, width: int, eps: float, streams: int):
        super().__init__()
        self.mixer = build_mixer(spec, width, eps)
        self.mlp = build_mlp(spec.mlp, width)
        self.hc1 = HyperConnection(width, streams, own_gate=False)
        self.hc2 = (HyperConnection(width, streams, own_gate=False)
                    if self.mlp is not None else None)


def cache_sources(layers: list) -> list:
    """Whose cache every layer reads: its own, or the earlier layer's whose
    latent rows it takes."""
    out = []
    for i, spec in enumerate(layers):
        src = spec.mixer.get("kv_from") if spec.type == "latent_attention" else None
        if src is None:
            out.append(i)
            continue
        src = int(src)
        if not 0 <= src < i:
            raise ValueError(f"layer {i}: kv_from must name an earlier layer")
        other = layers[src]
        if other.type != "latent_attention" or other.mixer.get("kv_from") is not None:
            raise ValueError(f"layer {i}: kv_from layer {src} caches no latent")
        for key in ("kv_rank", "rot_dim", "rot"):
            if other.mixer[key] != spec.mixer[key]:
                raise ValueError(f"layer {i}: {key} differs from layer {src}'s")
        out.append(src)
    return out


class LipulornForCausalLM(nn.Module):
    #: delta-rule layers carry state: the engine gives every live sequence a
    #: state slot and builds fb.seq
    has_seq_state = True

    def __init__(self, cfg: ModelArchConfig, device=None, dtype=torch.bfloat16):
        super().__init__()
        assert cfg.hybrid is not None
        self.cfg = cfg
        self.dtype = dtype
        hs = cfg.hybrid
        W = cfg.hidden_size
        self.eps = hs.norm_eps
        self.streams = int(hs.streams)
        prev_dtype = torch.get_default_dtype()
        torch.set_default_dtype(dtype)
        try:
            with torch.device(device if device is not None else "cpu"):
                self.embed_tokens = nn.Embedding(cfg.vocab_size, W)
                self.layers = nn.ModuleList(
                    [LipulornLayer(spec, W, hs.norm_eps, self.streams) for spec in hs.layers]
                )
                self.final_norm = _f32(W)
                nn.init.ones_(self.final_norm)
                self.final_read = _f32(self.streams)
                nn.init.ones_(self.final_read)  # the streams are summed at the end
                self.lm_head = nn.Parameter(torch.empty(cfg.vocab_size, W),
                                            requires_grad=False)
                nn.init.normal_(self.lm_head, std=W ** -0.5)
        finally:
            torch.set_default_dtype(prev_dtype)
        self.cache_of = cache_sources(hs.layers)
        self.capture_layers = None  # set to a list to record per-layer residuals

    # -- what the runner allocates per layer -----------------------------
    def kv_cache_specs(self):
        return [layer.mixer.kv_spec() for layer in self.layers]

    def state_specs(self):
        return [layer.mixer.state_spec() for layer in self.layers]

    def bind_kv_caches(self, kv_caches):
        self.kv_caches = [kv_caches[j] for j in self.cache_of]

    def bind_states(self, states):
        self.states = states

    # --------------------------------------------------------------------
    @torch.inference_mode()
    def forward(self, fb: ForwardBatch) -> torch.Tensor:
        X = sops.embed_streams(fb.input_ids, self.embed_tokens.weight,
                               self.streams)  # [T, S, C] fp32
        y = hc = None  # the sublayer output not yet written to the streams

        def read(rd, norm):
            return sops.hyper_mix_rmsnorm(
                X, y, None, hc.mix if hc is not None else None,
                hc.write if hc is not None else None, rd, norm, self.eps, self.dtype)

        for i, layer in enumerate(self.layers):
            h = read(layer.hc1.read, layer.hc1.norm)
            hc = layer.hc1
            y = layer.mixer(h, fb, self.states[i], self.kv_caches[i])
            if layer.mlp is not None:
                h = read(layer.hc2.read, layer.hc2.norm)
                hc = layer.hc2
                y = layer.mlp(h)
            if self.capture_layers is not None:
                self.capture_layers.append(hc.written(X, y).sum(1))
        return read(self.final_read, self.final_norm)

    @torch.inference_mode()
    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return F.linear(hidden, self.lm_head).float()

    # -- checkpoint names -> fused engine layout -----------------------------
    def load_named_tensors(self, tensors) -> int:
        """tensors: iterable of (name, tensor) with the design's names
        ('embed', 'l<i>.norm1', 'l<i>.hc1.in', 'l<i>.mix.a1', 'l<i>.mlp.up.b',
        'final.norm', 'head', ...)."""
        W = {k: v for k, v in tensors}
        used = set()

        def get(name):
            used.add(name)
            try:
                return W[name]
            except KeyError:
                raise ValueError(f"checkpoint lacks tensor {name!r}") from None

        def put(param, value):
            value = value.to(device=param.device, dtype=param.dtype)
            if param.shape != value.shape:
                raise ValueError(
                    f"checkpoint tensor of shape {tuple(value.shape)} does not fit "
                    f"{tuple(param.shape)}")
            param.data.copy_(value)

        def put_parts(param, parts):
            """Fill a parameter from {index: tensor}; what no part covers is
            zero."""
            full = torch.zeros(param.shape, dtype=param.dtype)
            for at, value in parts:
                if full[at].shape != value.shape:
                    raise ValueError(
                        f"checkpoint tensor of shape {tuple(value.shape)} does not fit "
                        f"{tuple(full[at].shape)}")
                full[at] = value.to(param.dtype)
            put(param, full)

        put(self.embed_tokens.weight, get("embed"))
        put(self.lm_head, get("head"))
        put(self.final_norm, get("final.norm"))
        for i, layer in enumerate(self.layers):
            p = f"l{i}."
            for n, hc in ((1, layer.hc1), (2, layer.hc2)):
                if hc is None:
                    continue
                put(hc.norm, get(f"{p}norm{n}"))
                put(hc.read, get(f"{p}hc{n}.in"))
                put(hc.write, get(f"{p}hc{n}.out"))
                put(hc.mix, get(f"{p}hc{n}.mix"))
            m, q = layer.mixer, p + "mix."
            if isinstance(m, HeadGatedAttention):
                rows = slice(0, sum(m.sizes))
                put_parts(m.in_proj.weight,
                          [(rows, torch.cat([get(q + n) for n in ("q", "k", "v", "g")]))])
                put_parts(m.in_proj.bias,
                          [(slice(0, sum(m.sizes[:3])),
                            torch.cat([get(q + n + ".b") for n in ("q", "k", "v")]))])
            elif isinstance(m, LatentAttention):
                H, D, Dv, R = m.heads, m.dim, m.vdim, m.rank
                parts = [get(q + "dq")]
                put(m.q_norm, get(q + "dq.norm"))
                put(m.q_up.weight, get(q + "uq"))
                if m.own_latent:
                    parts.append(get(q + "dkv"))
                    put(m.latent_norm, get(q + "dkv.norm"))
                put(m.in_proj.weight, torch.cat(parts))
                put(m.uk_r, get(q + "uk").reshape(H, D, R).transpose(1, 2))
                put(m.uv, get(q + "uv").reshape(H, Dv, R))
            else:
                a1, g1 = get(q + "a1"), get(q + "g1")
                m.set_ranks(a1.shape[0], g1.shape[0])
                put_parts(m.in_proj.weight, [
                    (m.at["qkv"], torch.cat([get(q + n) for n in ("q", "k", "v")])),
                    (m.at["low"], torch.cat([a1, g1])), (m.at["beta"], get(q + "b"))])
                put_parts(m.low_proj.weight, [
                    ((m.up_decay, slice(0, m.decay_rank)), get(q + "a2")),
                    ((m.up_gate, slice(m.decay_rank, None)), get(q + "g2"))])
                put(m.conv.weight, torch.cat([get(q + n + ".conv") for n in ("q", "k", "v")]))
                put(m.a_log, get(q + "A_log"))
                put(m.dt_bias, get(q + "dt_bias"))
                put(m.norm, get(q + "norm").repeat(m.heads))
            put(m.o_proj.weight, get(q + "o"))
            f, q = layer.mlp, p + "mlp."
            if f is None:
                continue
            put(f.gate_up.weight, torch.cat([get(q + "gate"), get(q + "up")]))
            put(f.gate_up.bias, torch.cat([get(q + "gate.b"), get(q + "up.b")]))
            put(f.down.weight, get(q + "down"))
            put(f.down.bias, get(q + "down.b"))
        missing = set(W) - used
        if missing:
            raise ValueError(f"checkpoint tensors not consumed: {sorted(missing)[:8]}")
        return len(used)
