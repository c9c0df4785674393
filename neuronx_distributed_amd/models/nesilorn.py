"""Nesilorn: a decoder of gated latent attention and mixtures of experts,
normed after every sublayer instead of before.

    x = scale * embed[token]
    per layer:  x <- x + norm1(mixer(x));  x <- x + norm2(mlp(x))  (if any)
    logits = embed norm(x)

The norm weights are stored as their distance from one.  The residual stream
is float32; a sublayer reads its rounding.  The pieces live in
``models/mixers.py`` and run on the serving kernels, through the serving
engine only.
"""

import dataclasses
from dataclasses import dataclass
from typing import List

import torch
import torch.nn as nn

from ..ops import serving as sv
from ..parallel import parallel_state as ps
from ..parallel.layers import ParallelEmbedding
from .mixers import (CheckpointReader, ExpertsMLP, GeluMLP, LatentAttention,
                     SingleMixer, copy_weight)


@dataclass
class NesilornConfig:
    vocab_size: int
    hidden_size: int
    layers: List[dict]          # type, mixer sizes, mlp or None — per layer
    norm_eps: float
    embedding_scale: float = 1.0

    @classmethod
    def from_dict(cls, d: dict) -> "NesilornConfig":
        return cls(vocab_size=d["vocab"], hidden_size=d["width"],
                   layers=d["layers"], norm_eps=d["norm"]["eps"],
                   embedding_scale=d["embedding"]["scale"])


def _latent_attention(width, c, eps):
    mask = c.get("mask") or {}
    return SingleMixer(width, LatentAttention(
        width, c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"],
        c["scale"], c["rot"]["base"], c["rot"]["dims"], eps,
        mask.get("size") or 0))


# of the experts' activation
GLU_ALPHA, GLU_SHIFT = 1.702, 1.0


def _experts(width, c):
    return ExpertsMLP(width, c["expert"]["ff"], c["router"]["experts"],
                      c["router"]["top"], c["expert"]["limit"], GLU_ALPHA,
                      GLU_SHIFT)


MIXERS = {"latent_attention": _latent_attention}
MLPS = {"dense": lambda width, c: GeluMLP(width, c["ff"]),
        "moe": _experts}


def _bench_layers(n, heads, dim, rot, vdim, rank, window, dense_ff, experts,
                  top, ff, first_dense=1):
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim,
             "kv_rank": rank, "scale": (dim + rot) ** -0.5,
             "rot": {"base": 1e4, "dims": rot}, "mask": {"size": window}}
    dense = {"kind": "dense", "ff": dense_ff}
    moe = {"kind": "moe", "router": {"experts": experts, "top": top},
           "expert": {"ff": ff, "limit": 7.0}}
    return [{"type": "latent_attention", "mixer": mixer,
             "mlp": dense if i < first_dense else moe} for i in range(n)]


NESILORN_CONFIGS = {
    # layer shapes of an 8-expert 7B-class decoder (random weights; for
    # timing)
    "nesilorn-bench": NesilornConfig(
        vocab_size=32000, hidden_size=4096, norm_eps=1e-5,
        embedding_scale=2.0,
        layers=_bench_layers(4, 32, 128, 64, 128, 512, 4096, 14336, 8, 2,
                             14336, 0)),
    # of many small experts
    "nesilorn-bench-fine": NesilornConfig(
        vocab_size=32000, hidden_size=2048, norm_eps=1e-5,
        embedding_scale=2.0,
        layers=_bench_layers(4, 16, 128, 64, 128, 512, 4096, 14336, 64, 6,
                             1408, 0)),
    "nesilorn-tiny": NesilornConfig(
        vocab_size=320, hidden_size=128, norm_eps=1e-5, embedding_scale=2.0,
        layers=_bench_layers(3, 2, 24, 16, 40, 48, 50, 160, 6, 2, 72)),
}


def get_nesilorn_config(name: str, **overrides) -> NesilornConfig:
    return dataclasses.replace(NESILORN_CONFIGS[name], **overrides)


class NesilornLayer(nn.Module):
    def __init__(self, config: NesilornConfig, layer: dict):
        super().__init__()
        width = config.hidden_size
        mlp = layer.get("mlp")
        for kind, known in ((layer["type"], MIXERS),
                            ((mlp or {}).get("kind", "dense"), MLPS)):
            if kind not in known:
                raise ValueError(f"unknown layer kind {kind!r}; this model "
                                 f"has {sorted(known)}")
        self.eps = config.norm_eps
        self.norm1 = nn.Parameter(torch.zeros(width))
        self.mix = MIXERS[layer["type"]](width, layer["mixer"], self.eps)
        self.mlp = None
        if mlp is not None:
            self.norm2 = nn.Parameter(torch.zeros(width))
            self.mlp = MLPS[mlp.get("kind", "dense")](width, mlp)

    def load(self, get, prefix):
        copy_weight(self.norm1, get(prefix + "norm1"))
        self.mix.load(get, prefix + "mix.")
        if self.mlp is not None:
            copy_weight(self.norm2, get(prefix + "norm2"))
            self.mlp.load(get, prefix + "mlp.")

    def _read(self, x, pending):
        """Add what is pending; the stream and its rounding."""
        x, h, _ = sv.residual_norm(x, pending, self.eps, copy=True,
                                   dtype=self.norm1.dtype)
        return x, h

    def forward(self, x, pending, batch, pools):
        """(x, pending) -> (x, pending): the stream is x + pending; the norm
        of a sublayer's output and the residual add are one kernel."""
        x, h = self._read(x, pending)
        pending = self.mix(h, batch, pools)
        pending.w1, pending.centred = self.norm1, True
        if self.mlp is not None:
            x, h = self._read(x, pending)
            pending = self.mlp(h)
            pending.w1, pending.centred = self.norm2, True
        return x, pending


class NesilornForCausalLM(nn.Module):
    """Served through ``inference.InferenceEngine`` (``forward_ragged``)."""
    supports_ragged = True

    def __init__(self, config: NesilornConfig):
        super().__init__()
        if ps.get_tensor_model_parallel_size() != 1:
            raise NotImplementedError(
                "Nesilorn is served one model per GPU (all heads share one "
                "latent); tensor parallelism is not implemented")
        self.config = config
        self.embed = ParallelEmbedding(config.vocab_size, config.hidden_size)
        self.layers = nn.ModuleList(NesilornLayer(config, l)
                                    for l in config.layers)
        self.final_norm = nn.Parameter(torch.zeros(config.hidden_size))

    def load_checkpoint(self, tensors: dict):
        """Fill every parameter from a name -> tensor dictionary; a missing,
        unused or misshapen tensor is an error."""
        get = CheckpointReader(tensors)
        copy_weight(self.embed.weight, get("embed"))
        for i, layer in enumerate(self.layers):
            layer.load(get, f"l{i}.")
        copy_weight(self.final_norm, get("final.norm"))
        get.done()

    def cache_specs(self):
        return [layer.mix.cache_specs() for layer in self.layers]

    def forward_ragged(self, batch, pools):
        """Packed step -> float32 logits (wanted, vocab), or None."""
        x, pending = None, sv.Pending(self.embed(batch.tokens),
                                      scale=self.config.embedding_scale)
        for layer, pool in zip(self.layers, pools):
            x, pending = layer(x, pending, batch, pool)
        if not batch.want.shape[0]:
            return None
        _, h, _ = sv.residual_norm(x, pending, self.config.norm_eps,
                                   self.final_norm, keep_x=False,
                                   index=batch.want, centred=True)
        return sv.linear_f32(h, self.embed.weight)

    def forward(self, *args, **kwargs):
        raise NotImplementedError("Nesilorn runs through the serving engine: "
                                  "inference.generate or InferenceEngine")
