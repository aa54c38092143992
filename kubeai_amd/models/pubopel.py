"""Pubopel: a decoder without a single statistic in its layer norms. Every
sublayer is bracketed by two dynamic tanh, dyt(x) = tanh(alpha x) * w + b,

    x <- x + dyt_b(sublayer(h + conv(h))),   h = dyt_a(x),

where conv is a causal convolution over time on each channel, whose last
taps - 1 inputs are state of the sequence, for both sublayers of every layer.
The mixer is softmax attention whose values are its keys (one cached row per
token serves as both), with whole-projection q/k RMS norms, per-head score
multipliers, a tanh cap, a distance bias, a learned sink and an optional
sliding window behind which the first tokens stay visible; the feed-forward
is a mixture of gated experts that read the token times its own sigmoid
score, plus a shared expert (kubeai_amd.models.mixers).

Same execution model as the other layer-list decoders: one token-packed
forward per engine step, GEMMs through the BLAS library in the serving dtype,
everything else in the gfx950 kernels of kubeai_amd.ops.seq. The residual is
fp32; since dyt is elementwise, a sublayer's post-norm, the residual add, the
next pre-norm, its convolution and the advance of the carried tail are one
kernel.
"""
from __future__ import annotations

import torch
import torch.nn as nn
import torch.nn.functional as F

from kubeai_amd.engine.batch import ForwardBatch
from kubeai_amd.ops import seq as sops
from .config import HybridLayerSpec, ModelArchConfig
from .mixers import CausalConvTails, RoutedGatedMoE, TiedValueAttention, _f32


def distance_slopes(heads: int) -> list:
    """2^(-8 (h + 1) / heads): the bias per position of every head."""
    return [2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)]


def build_mixer(spec: HybridLayerSpec, width: int, eps: float) -> nn.Module:
    m = spec.mixer
    if spec.type != "attention":
        raise ValueError(f"unknown mixer type {spec.type!r}")
    heads, dim = int(m["heads"]), int(m["dim"])
    if int(m.get("vdim", dim)) != dim:
        raise ValueError("the values are the keys: vdim must equal dim")
    mask = m.get("mask") or {}
    if mask and int(mask["size"]) < 1:
        raise ValueError("a window must hold at least the token itself")
    return TiedValueAttention(
        width, heads=heads, kv_heads=int(m.get("kv_heads", heads)), dim=dim,
        scale=m["scale"], softcap=m.get("softcap") or 0.0,
        window=int(mask.get("size", 0)), keep_first=int(mask.get("keep_first") or 0),
        slopes=distance_slopes(heads), sink=True, eps=eps,
    )


def build_mlp(mlp: dict | None, width: int):
    if mlp is None:
        return None
    if mlp.get("kind", "moe") != "moe":
        raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
    return RoutedGatedMoE(
        width, experts=int(mlp["router"]["experts"]), top=int(mlp["router"]["top"]),
        ff=int(mlp["expert"]["ff"]), correction=False,
        shared_ff=int((mlp.get("shared") or {}).get("ff", 0)), score="sigmoid",
        weight_on="input",
    )


class DynTanh(nn.Module):
    """tanh(alpha x) * weight + bias, all parameters fp32."""

    def __init__(self, width: int):
        super().__init__()
        self.alpha, self.weight, self.bias = _f32(1), _f32(width), _f32(width)
        nn.init.constant_(self.alpha, 0.5)
        nn.init.ones_(self.weight)

    @property
    def params(self):
        return self.alpha, self.weight, self.bias


class PubopelLayer(nn.Module):
    def __init__(self, spec: HybridLayerSpec, width: int, eps: float, taps: int):
        super().__init__()
        self.mixer = build_mixer(spec, width, eps)
        self.mlp = build_mlp(spec.mlp, width)
        self.norm1, self.norm1b = DynTanh(width), DynTanh(width)
        self.canon1 = CausalConvTails(width, taps, residual=True)
        if self.mlp is not None:
            self.norm2, self.norm2b = DynTanh(width), DynTanh(width)
            self.canon2 = CausalConvTails(width, taps, residual=True)

    def state_spec(self):
        spec = dict(self.mixer.state_spec())
        spec["canon1"] = self.canon1.state_shape()
        if self.mlp is not None:
            spec["canon2"] = self.canon2.state_shape()
        return spec


class PubopelForCausalLM(nn.Module):
    #: the input convolutions carry state: the engine gives every live
    #: sequence a state slot and builds fb.seq
    has_seq_state = True

    def __init__(self, cfg: ModelArchConfig, device=None, dtype=torch.bfloat16):
        super().__init__()
        assert cfg.hybrid is not None
        self.cfg = cfg
        self.dtype = dtype
        hs = cfg.hybrid
        W = cfg.hidden_size
        prev_dtype = torch.get_default_dtype()
        torch.set_default_dtype(dtype)
        try:
            with torch.device(device if device is not None else "cpu"):
                self.embed_tokens = nn.Embedding(cfg.vocab_size, W)
                self.layers = nn.ModuleList(
                    [PubopelLayer(spec, W, hs.norm_eps, hs.canon_taps) for spec in hs.layers]
                )
                self.final_norm = DynTanh(W)
                self.lm_head = nn.Parameter(torch.empty(cfg.vocab_size, W),
                                            requires_grad=False)
                nn.init.normal_(self.lm_head, std=W ** -0.5)
        finally:
            torch.set_default_dtype(prev_dtype)
        self.capture_layers = None  # set to a list to record per-layer residuals

    # -- what the runner allocates per layer -----------------------------
    def kv_cache_specs(self):
        return [layer.mixer.kv_spec() for layer in self.layers]

    def state_specs(self):
        return [layer.state_spec() for layer in self.layers]

    def bind_kv_caches(self, kv_caches):
        self.kv_caches = kv_caches

    def bind_states(self, states):
        self.states = states

    # --------------------------------------------------------------------
    @torch.inference_mode()
    def forward(self, fb: ForwardBatch) -> torch.Tensor:
        residual = self.embed_tokens(fb.input_ids.long()).float()
        y = post = None  # the sublayer output not yet added, and its norm

        def advance(pre, canon=None, tails=None):
            return sops.add_dyt_conv(
                y, post.params if post is not None else None, residual, pre.params,
                canon.weight if canon is not None else None, tails, fb.seq, self.dtype)

        for i, layer in enumerate(self.layers):
            state = self.states[i]
            h, residual = advance(layer.norm1, layer.canon1, state["canon1"])
            if self.capture_layers is not None and i > 0:
                self.capture_layers.append(residual.clone())
            y, post = layer.mixer(h, fb, state, self.kv_caches[i]), layer.norm1b
            if layer.mlp is not None:
                h, residual = advance(layer.norm2, layer.canon2, state["canon2"])
                y, post = layer.mlp(h), layer.norm2b
        h, residual = advance(self.final_norm)
        if self.capture_layers is not None:
            self.capture_layers.append(residual.clone())
        return h

    @torch.inference_mode()
    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return F.linear(hidden, self.lm_head).float()

    # -- checkpoint names -> fused engine layout -----------------------------
    def load_named_tensors(self, tensors) -> int:
        """tensors: iterable of (name, tensor) with the design's names
        ('embed', 'l<i>.norm1', 'l<i>.norm1.alpha', 'l<i>.canon1',
        'l<i>.mix.q', 'l<i>.mlp.e<k>.gate', 'final.norm', 'head', ...)."""
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

        def put_dyt(norm, name):
            put(norm.alpha, get(name + ".alpha").reshape(1))
            put(norm.weight, get(name))
            put(norm.bias, get(name + ".b"))

        put(self.embed_tokens.weight, get("embed"))
        put(self.lm_head, get("head"))
        put_dyt(self.final_norm, "final.norm")
        for i, layer in enumerate(self.layers):
            p = f"l{i}."
            put_dyt(layer.norm1, p + "norm1")
            put_dyt(layer.norm1b, p + "norm1b")
            put(layer.canon1.weight, get(p + "canon1"))
            m, q = layer.mixer, p + "mix."
            put(m.in_proj.weight, torch.cat([get(q + "q"), get(q + "k")]))
            put(m.q_weight, m.fold_query_weight(get(q + "q.norm"), get(q + "k.norm"),
                                                get(q + "temp")))
            put(m.sink_scores, get(q + "sink"))
            put(m.o_proj.weight, get(q + "o"))
            f, q = layer.mlp, p + "mlp."
            if f is None:
                continue
            put_dyt(layer.norm2, p + "norm2")
            put_dyt(layer.norm2b, p + "norm2b")
            put(layer.canon2.weight, get(p + "canon2"))
            names = [f"{q}e{e}." for e in range(f.experts)]
            if f.shared_ff:
                names.append(q + "shared.")
            put(f.gate_up.weight,
                torch.cat([get(n + part) for n in names for part in ("gate", "up")]))
            put(f.down.weight, torch.cat([get(n + "down") for n in names], dim=1))
            put(f.router, get(q + "router"))
        missing = set(W) - used
        if missing:
            raise ValueError(f"checkpoint tensors not consumed: {sorted(missing)[:8]}")
        return len(used)
