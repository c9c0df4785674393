"""Voletar: a decoder that interleaves matrix memories with parallel
attention/memory layers and runs a block of its layers several times.

    x  = embed[token]                                  (x0)
    per pass of the looped block:  x <- W_in [x; x0] + step[pass]
    per layer:  x <- x + mixer(norm1 x);  x <- x + mlp(norm2 x)  (if any)
    logits = cap tanh(head norm(x) / cap)

Mixers: ``lightning`` (DecayMemory) and ``parallel`` (SlidingAttention beside
GatedMemory).  The residual stream is float32; the pieces live in
``models/mixers.py`` and run on the serving kernels, through the serving
engine only.
"""

import dataclasses
import math
from dataclasses import dataclass
from typing import List, Optional

import torch
import torch.nn as nn

from ..ops import serving as sv
from ..parallel import parallel_state as ps
from ..parallel.layers import ColumnParallelLinear, ParallelEmbedding
from .mixers import (CheckpointReader, DecayMemory, GatedMemory, ParallelMixer,
                     ReluSquaredMLP, SingleMixer, SlidingAttention,
                     copy_weight)


@dataclass
class VoletarConfig:
    vocab_size: int
    hidden_size: int
    layers: List[dict]          # type, mixer sizes, mlp or None — per layer
    norm_eps: float
    logit_softcap: float
    loop: Optional[dict] = None  # start, stop, times

    @classmethod
    def from_dict(cls, d: dict) -> "VoletarConfig":
        return cls(vocab_size=d["vocab"], hidden_size=d["width"],
                   layers=d["layers"], norm_eps=d["norm"]["eps"],
                   logit_softcap=d["logit_softcap"], loop=d.get("loop"))

    def schedule(self):
        """(layer, pass) of every layer run, in order; the pass is given at
        the first layer of each pass of the looped block, else None."""
        n = len(self.layers)
        if not self.loop:
            return [(i, None) for i in range(n)]
        a, b = self.loop["start"], self.loop["stop"]
        if not 0 <= a < b <= n:
            raise ValueError(f"looped layers {a}..{b} of {n}")
        runs = [(i, None) for i in range(a)]
        for t in range(self.loop["times"]):
            runs += [(i, t if i == a else None) for i in range(a, b)]
        return runs + [(i, None) for i in range(b, n)]


def _lightning(width, c, eps):
    return SingleMixer(width, DecayMemory(
        width, c["heads"], c["dim"], c["vdim"], c["decay"], eps))


def _parallel(width, c, eps):
    l, r = c["left"], c["right"]
    mask = l.get("mask") or {}
    return ParallelMixer(
        width,
        SlidingAttention(width, l["heads"], l["kv_heads"], l["dim"],
                         l["vdim"], l["scale"], mask.get("size", 0),
                         mask.get("keep_first", 0)),
        GatedMemory(width, r["heads"], r["dim"], r["vdim"], r["gate_cap"],
                    eps))


MIXERS = {"lightning": _lightning, "parallel": _parallel}
MLPS = {"dense": lambda width, c: ReluSquaredMLP(width, c["ff"])}


def _bench_layers(n, width, heads, kv_heads, dim, window, keep, m_heads,
                  m_dim, m_vdim, ff):
    light = {"type": "lightning", "mlp": None, "mixer": {
        "heads": heads, "dim": dim, "vdim": dim,
        "decay": [math.exp(-2.0 ** (-8.0 * (h + 1) / heads))
                  for h in range(heads)]}}
    par = {"type": "parallel", "mlp": {"kind": "dense", "ff": ff}, "mixer": {
        "left": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                 "vdim": dim, "scale": dim ** -0.5,
                 "mask": {"size": window, "keep_first": keep}},
        "right": {"heads": m_heads, "dim": m_dim, "vdim": m_vdim,
                  "gate_cap": 15.0}}}
    return [light if i % 2 == 0 else par for i in range(n)]


VOLETAR_CONFIGS = {
    # layer shapes of a 7B-class decoder (random weights; for timing)
    "voletar-bench": VoletarConfig(
        vocab_size=32000, hidden_size=4096, norm_eps=1e-6,
        logit_softcap=50.0, loop={"start": 0, "stop": 2, "times": 2},
        layers=_bench_layers(4, 4096, 32, 8, 128, 4096, 64, 16, 128, 256,
                             14336)),
    "voletar-tiny": VoletarConfig(
        vocab_size=320, hidden_size=128, norm_eps=1e-5, logit_softcap=20.0,
        loop={"start": 1, "stop": 3, "times": 3},
        layers=_bench_layers(4, 128, 2, 1, 32, 48, 9, 2, 16, 40, 160)),
}


def get_voletar_config(name: str, **overrides) -> VoletarConfig:
    return dataclasses.replace(VOLETAR_CONFIGS[name], **overrides)


class VoletarLayer(nn.Module):
    def __init__(self, config: VoletarConfig, layer: dict):
        super().__init__()
        width = config.hidden_size
        for kind, known in ((layer["type"], MIXERS),
                            ((layer["mlp"] or {}).get("kind", "dense"),
                             MLPS)):
            if kind not in known:
                raise ValueError(f"unknown layer kind {kind!r}; this model "
                                 f"has {sorted(known)}")
        self.norm1 = nn.Parameter(torch.ones(width))
        self.mix = MIXERS[layer["type"]](width, layer["mixer"],
                                         config.norm_eps)
        self.mlp = None
        if layer["mlp"] is not None:
            self.norm2 = nn.Parameter(torch.ones(width))
            self.mlp = MLPS[layer["mlp"].get("kind", "dense")](width,
                                                               layer["mlp"])

    def load(self, get, prefix):
        copy_weight(self.norm1, get(prefix + "norm1"))
        self.mix.load(get, prefix + "mix.")
        if self.mlp is not None:
            copy_weight(self.norm2, get(prefix + "norm2"))
            self.mlp.load(get, prefix + "mlp.")

    def forward(self, x, pending, eps, batch, pools):
        """(x, pending) -> (x, pending): the stream is x + pending; every
        residual add fuses into the norm that follows it."""
        x, h, _ = sv.residual_norm(x, pending, eps, self.norm1)
        pending = self.mix(h, batch, pools)
        if self.mlp is not None:
            x, h, _ = sv.residual_norm(x, pending, eps, self.norm2)
            pending = self.mlp(h)
        return x, pending


class VoletarForCausalLM(nn.Module):
    """Served through ``inference.InferenceEngine`` (``forward_ragged``)."""
    supports_ragged = True

    def __init__(self, config: VoletarConfig):
        super().__init__()
        if ps.get_tensor_model_parallel_size() != 1:
            raise NotImplementedError(
                "Voletar is served one model per GPU (its lightning norm "
                "spans all heads); tensor parallelism is not implemented")
        self.config = config
        W = config.hidden_size
        self.embed = ParallelEmbedding(config.vocab_size, W)
        self.layers = nn.ModuleList(VoletarLayer(config, l)
                                    for l in config.layers)
        self.runs = config.schedule()
        if config.loop:
            self.loop_in = nn.Parameter(
                torch.randn(W, 2 * W) * (2 * W) ** -0.5)
            self.loop_step = nn.Parameter(
                torch.zeros(config.loop["times"], W))
        self.final_norm = nn.Parameter(torch.ones(W))
        self.head = ColumnParallelLinear(W, config.vocab_size, bias=False,
                                         gather_output=False)

    def load_checkpoint(self, tensors: dict):
        """Fill every parameter from a name -> tensor dictionary; a missing,
        unused or misshapen tensor is an error."""
        get = CheckpointReader(tensors)
        copy_weight(self.embed.weight, get("embed"))
        if self.config.loop:
            copy_weight(self.loop_in, get("loop.in"))
            copy_weight(self.loop_step, get("loop.step"))
        for i, layer in enumerate(self.layers):
            layer.load(get, f"l{i}.")
        copy_weight(self.final_norm, get("final.norm"))
        copy_weight(self.head.weight, get("head"))
        get.done()

    def cache_specs(self):
        """What each layer run keeps; every pass of a looped layer has its
        own."""
        return [self.layers[i].mix.cache_specs() for i, _ in self.runs]

    def forward_ragged(self, batch, pools):
        """Packed step -> float32 logits (wanted, vocab), or None."""
        eps = self.config.norm_eps
        x0 = self.embed(batch.tokens)
        x, pending = None, sv.Pending(x0)
        for (i, t), pool in zip(self.runs, pools):
            if t is not None:
                _, _, cat = sv.residual_norm(x, pending, eps, x0=x0,
                                             keep_x=False)
                x, pending = None, sv.Pending(
                    sv.linear_f32(cat, self.loop_in), vec=self.loop_step[t])
            x, pending = self.layers[i](x, pending, eps, batch, pool)
        if not batch.want.shape[0]:
            return None
        _, h, _ = sv.residual_norm(x, pending, eps, self.final_norm,
                                   keep_x=False, index=batch.want)
        return sv.softcap_(sv.linear_f32(h, self.head.weight),
                           self.config.logit_softcap)

    def forward(self, *args, **kwargs):
        raise NotImplementedError("Voletar runs through the serving engine: "
                                  "inference.generate or InferenceEngine")
