"""Sutuvik: a decoder of state-space memories and two kinds of modified
attention, with mixtures of experts and a per-layer token input.

    x = norm(embed[token])
    per layer:  h = norm1(x);  x <- x + mixer(h + conv(h))
                x <- x + mlp(norm2(x))  (if any)
                x <- x + side(x, token)
    logits = scale * embed norm(x)

The model's norm runs in groups of the width; conv is a short causal
convolution a channel.  The residual stream is float32.  The pieces live in
``models/mixers.py`` and run on the serving kernels, through the serving engine
only.
"""

import dataclasses
from dataclasses import dataclass
from typing import List

import torch
import torch.nn as nn

from ..inference.paged_cache import ConvRing
from ..ops import serving as sv
from ..parallel import parallel_state as ps
from ..parallel.layers import ParallelEmbedding
from .mixers import (CheckpointReader, ExpertsMLP, ScoredAttention,
                     SingleMixer, StateSpaceMemory, TokenSide, alibi_slopes,
                     copy_weight)


@dataclass
class SutuvikConfig:
    vocab_size: int
    hidden_size: int
    layers: List[dict]          # type, mixer sizes, mlp or None — per layer
    norm_eps: float
    norm_groups: int
    conv_taps: int
    side_dim: int
    logit_scale: float = 1.0

    @classmethod
    def from_dict(cls, d: dict) -> "SutuvikConfig":
        return cls(vocab_size=d["vocab"], hidden_size=d["width"],
                   layers=d["layers"], norm_eps=d["norm"]["eps"],
                   norm_groups=d["norm"]["groups"],
                   conv_taps=d["canon"]["taps"],
                   side_dim=d["token_side"]["dim"],
                   logit_scale=d.get("logit_scale", 1.0))


def _mamba2(width, c, eps):
    return SingleMixer(width, StateSpaceMemory(
        width, c["heads"], c["vdim"], c["state"], c["groups"], c["conv"],
        c["norm_groups"], eps))


def _attention(width, c, eps):
    return SingleMixer(width, ScoredAttention(
        width, c["heads"], c["kv_heads"], c["dim"], c["vdim"], c["scale"],
        eps, qk_norm="weighted", q_temp=c.get("q_temp"),
        slopes=alibi_slopes(c["heads"]), sink="learned", gate=True,
        v_mix=bool(c.get("v_mix"))))


def _attention_2(width, c, eps):
    return SingleMixer(width, ScoredAttention(
        width, c["heads"], c["kv_heads"], c["dim"], c["vdim"], c["scale"],
        eps, rot=c.get("rot"), qk_norm="plain", head_temp=True,
        softcap=c.get("softcap"), sink="zero", v_mix=bool(c.get("v_mix"))))


def _experts(width, c):
    r = c["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    return ExpertsMLP(width, c["expert"]["ff"], r["experts"],
                      sv.Routing(r["top"], True, g["count"], g["keep"]),
                      bias_name="correction")


MIXERS = {"mamba2": _mamba2, "attention": _attention,
          "attention_2": _attention_2}
MLPS = {"moe": _experts}


def _bench_layers(order, m_heads, m_vdim, state, groups, heads, kv_heads, dim,
                  experts, top, count, keep, ff):
    mixers = {
        "mamba2": {"heads": m_heads, "vdim": m_vdim, "state": state,
                   "groups": groups, "conv": 4, "norm_groups": groups},
        "attention": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                      "vdim": dim, "scale": dim ** -0.5, "v_mix": True,
                      "q_temp": {"coef": 0.1, "every": 8192}},
        "attention_2": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                        "vdim": dim, "scale": dim ** -0.5, "v_mix": True,
                        "softcap": 50.0,
                        "rot": {"base": 5e5, "dims": dim, "scaling": {
                            "factor": 8.0, "low": 1.0, "high": 4.0,
                            "original": 8192}}}}
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {
        "experts": experts, "top": top,
        "groups": {"count": count, "keep": keep}}}
    return [{"type": t, "mixer": mixers[t], "mlp": mlp} for t in order]


_ORDER = ("mamba2", "attention", "mamba2", "attention_2")

SUTUVIK_CONFIGS = {
    # layer shapes of an 8-expert 7B-class decoder (random weights; for
    # timing)
    "sutuvik-bench": SutuvikConfig(
        vocab_size=32000, hidden_size=4096, norm_eps=1e-5, norm_groups=8,
        conv_taps=4, side_dim=256, logit_scale=0.5,
        layers=_bench_layers(_ORDER, 128, 64, 128, 8, 32, 8, 128, 8, 2, 4, 2,
                             14336)),
    # of many small experts in groups
    "sutuvik-bench-fine": SutuvikConfig(
        vocab_size=32000, hidden_size=2048, norm_eps=1e-5, norm_groups=8,
        conv_taps=4, side_dim=128, logit_scale=0.5,
        layers=_bench_layers(_ORDER, 64, 64, 128, 4, 16, 4, 128, 64, 6, 8, 3,
                             1408)),
    "sutuvik-tiny": SutuvikConfig(
        vocab_size=320, hidden_size=128, norm_eps=1e-5, norm_groups=2,
        conv_taps=3, side_dim=16, logit_scale=0.5,
        layers=_bench_layers(_ORDER, 4, 32, 24, 2, 4, 2, 32, 8, 2, 4, 2, 72)),
}


def get_sutuvik_config(name: str, **overrides) -> SutuvikConfig:
    return dataclasses.replace(SUTUVIK_CONFIGS[name], **overrides)


class SutuvikLayer(nn.Module):
    def __init__(self, config: SutuvikConfig, layer: dict, index: int):
        super().__init__()
        width = config.hidden_size
        mlp = layer.get("mlp")
        for kind, known in ((layer["type"], MIXERS),
                            ((mlp or {}).get("kind", "moe"), MLPS)):
            if kind not in known:
                raise ValueError(f"unknown layer kind {kind!r}; this model "
                                 f"has {sorted(known)}")
        self.eps, self.groups = config.norm_eps, config.norm_groups
        self.norm1 = nn.Parameter(torch.ones(width))
        self.conv = nn.Parameter(torch.zeros(config.conv_taps, width))
        self.mix = MIXERS[layer["type"]](width, layer["mixer"], self.eps)
        self.mlp = None
        if mlp is not None:
            self.norm2 = nn.Parameter(torch.ones(width))
            self.mlp = MLPS[mlp.get("kind", "moe")](width, mlp)
        self.side = TokenSide(width, config.side_dim, index)
        # of layers whose values are mixed
        self.shares_values = getattr(self.mix.mixer, "v_mix", False)

    def cache_specs(self):
        return [ConvRing(self.conv.shape[1], self.conv.shape[0])] + \
            self.mix.cache_specs()

    def load(self, get, prefix):
        copy_weight(self.norm1, get(prefix + "norm1"))
        copy_weight(self.conv, get(prefix + "canon1").t())
        self.mix.load(get, prefix + "mix.")
        if self.mlp is not None:
            copy_weight(self.norm2, get(prefix + "norm2"))
            self.mlp.load(get, prefix + "mlp.")
        else:
            get.skip(prefix + "norm2")
        self.side.load(get, prefix + "side.")

    def forward(self, x, pending, table, values, batch, pools):
        """(x, pending) -> (x, pending): the stream is x + pending; every
        residual add fuses into the norm or the read that follows it."""
        x, h, _ = sv.residual_norm(
            x, pending, self.eps, self.norm1, groups=self.groups,
            conv=sv.ShortConv(self.conv, pools[0]), batch=batch)
        shared = {"values": values} if self.shares_values else {}
        pending = self.mix(h, batch, pools[1:], **shared)
        if self.mlp is not None:
            x, h, _ = sv.residual_norm(x, pending, self.eps, self.norm2,
                                       groups=self.groups)
            pending = self.mlp(h)
        x, h, _ = sv.residual_norm(x, pending, self.eps, copy=True,
                                   dtype=self.norm1.dtype)
        return x, self.side(h, table, batch.tokens)


class SutuvikForCausalLM(nn.Module):
    """Served through ``inference.InferenceEngine`` (``forward_ragged``)."""
    supports_ragged = True

    def __init__(self, config: SutuvikConfig):
        super().__init__()
        if ps.get_tensor_model_parallel_size() != 1:
            raise NotImplementedError(
                "Sutuvik is served one model per GPU (its norms span groups "
                "of the width); tensor parallelism is not implemented")
        W = config.hidden_size
        if W % config.norm_groups:
            raise ValueError(f"a width of {W} in {config.norm_groups} groups")
        if not 1 <= config.conv_taps <= sv.MAX_TAPS:
            raise ValueError(f"{config.conv_taps} taps")
        self.config = config
        self.embed = ParallelEmbedding(config.vocab_size, W)
        self.embed_norm = nn.Parameter(torch.ones(W))
        self.side_embed = nn.Parameter(torch.randn(
            config.vocab_size, len(config.layers) * config.side_dim))
        self.layers = nn.ModuleList(SutuvikLayer(config, l, i)
                                    for i, l in enumerate(config.layers))
        self.final_norm = nn.Parameter(torch.ones(W))

    def load_checkpoint(self, tensors: dict):
        """Fill every parameter from a name -> tensor dictionary; a missing,
        unused or misshapen tensor is an error."""
        get = CheckpointReader(tensors)
        copy_weight(self.embed.weight, get("embed"))
        copy_weight(self.embed_norm, get("embed.norm"))
        copy_weight(self.side_embed, get("side.embed"))
        for i, layer in enumerate(self.layers):
            layer.load(get, f"l{i}.")
        copy_weight(self.final_norm, get("final.norm"))
        get.done()

    def cache_specs(self):
        return [layer.cache_specs() for layer in self.layers]

    def forward_ragged(self, batch, pools):
        """Packed step -> float32 logits (wanted, vocab), or None."""
        c = self.config
        x, pending = None, sv.Pending(self.embed(batch.tokens),
                                      w1=self.embed_norm,
                                      groups=c.norm_groups)
        values = []          # of the first layer that mixes values
        for layer, pool in zip(self.layers, pools):
            x, pending = layer(x, pending, self.side_embed, values, batch,
                               pool)
        if not batch.want.shape[0]:
            return None
        _, h, _ = sv.residual_norm(x, pending, c.norm_eps, self.final_norm,
                                   keep_x=False, index=batch.want,
                                   groups=c.norm_groups, scale=c.logit_scale)
        return sv.linear_f32(h, self.embed.weight)

    def forward(self, *args, **kwargs):
        raise NotImplementedError("Sutuvik runs through the serving engine: "
                                  "inference.generate or InferenceEngine")
