"""Pokepel: a decoder of latent attention and retention layers, the mixer and the
feed-forward of a layer side by side.

    x = embed[token]
    per layer:  h = norm1(x)
                x <- x + sigmoid(R1 h + b1) * mixer(h)
                       + sigmoid(R2 h + b2) * mlp(h)     (if any)
    logits = head norm(x)

The residual stream is float32; both gated results are added by the kernel that
makes the next layer's h.  The pieces live in ``models/mixers.py`` and run on
the serving kernels, through the serving engine only.
"""

import dataclasses
from dataclasses import dataclass
from typing import List

import torch
import torch.nn as nn

from ..ops import serving as sv
from ..parallel import parallel_state as ps
from ..parallel.layers import ParallelEmbedding
from .mixers import (CheckpointReader, ExpertsMLP, GatedParallel,
                     LatentAttention, PolyNormMLP, Retention,
                     SharedExpertsMLP, copy_weight)


@dataclass
class PokepelConfig:
    vocab_size: int
    hidden_size: int
    layers: List[dict]          # type, mixer sizes, mlp or None — per layer
    norm_eps: float

    @classmethod
    def from_dict(cls, d: dict) -> "PokepelConfig":
        return cls(vocab_size=d["vocab"], hidden_size=d["width"],
                   layers=d["layers"], norm_eps=d["norm"]["eps"])


def _latent_attention(width, c, eps):
    rot = c["rot"]
    return LatentAttention(
        width, c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"],
        c["scale"], rot["base"], rot["dims"], eps, pairs=True,
        scaling=rot.get("scaling"), sink=True)


def _retention(width, c, eps):
    rot = c["rot"]
    return Retention(width, c["heads"], c["dim"], c["vdim"], c["decay"], eps,
                     rot["base"], rot["dims"], rot.get("scaling"))


def _dense(width, c, eps):
    return PolyNormMLP(width, c["ff"], eps)


def _experts(width, c, eps):
    r = c["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    return SharedExpertsMLP(width, ExpertsMLP(
        width, c["expert"]["ff"], r["experts"],
        sv.Routing(r["top"], groups=g["count"], keep=g["keep"], softmax=True,
                   best=1),
        bias_name=None), (c.get("shared") or {"ff": 0})["ff"])


MIXERS = {"latent_attention": _latent_attention, "retention": _retention}
MLPS = {"dense": _dense, "moe": _experts}


def _bench_layers(order, heads, dim, rot, vdim, rank, r_heads, r_dim, r_vdim,
                  experts, top, count, keep, ff, shared, dense_ff=None):
    mixers = {
        "latent_attention": {
            "heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim,
            "kv_rank": rank, "scale": (dim + rot) ** -0.5,
            "rot": {"base": 1e4, "dims": rot, "scaling": {
                "factor": 4.0, "fast": 32.0, "slow": 1.0,
                "original": 4096}}},
        "retention": {
            "heads": r_heads, "dim": r_dim, "vdim": r_vdim,
            "decay": [1.0 - 2.0 ** (-5.0 - 3.0 * h / r_heads)
                      for h in range(r_heads)],
            "rot": {"base": 1e4, "dims": r_dim}}}
    moe = {"kind": "moe", "expert": {"ff": ff}, "shared": {"ff": shared},
           "router": {"experts": experts, "top": top,
                      "groups": {"count": count, "keep": keep}}}
    return [{"type": t, "mixer": mixers[t],
             "mlp": {"kind": "dense", "ff": dense_ff}
             if dense_ff and i == 0 else moe} for i, t in enumerate(order)]


_ORDER = ("latent_attention", "retention", "latent_attention", "retention")

POKEPEL_CONFIGS = {
    # layer shapes of an 8-expert 7B-class decoder (random weights; for
    # timing)
    "pokepel-bench": PokepelConfig(
        vocab_size=32000, hidden_size=4096, norm_eps=1e-5,
        layers=_bench_layers(_ORDER, 32, 128, 64, 128, 512, 32, 128, 128, 8, 2,
                             4, 2, 14336, 4096)),
    # of many small experts in groups
    "pokepel-bench-fine": PokepelConfig(
        vocab_size=32000, hidden_size=2048, norm_eps=1e-5,
        layers=_bench_layers(_ORDER, 16, 128, 64, 128, 512, 16, 128, 128, 64,
                             6, 8, 3, 1408, 2816)),
    "pokepel-tiny": PokepelConfig(
        vocab_size=320, hidden_size=128, norm_eps=1e-5,
        layers=_bench_layers(_ORDER, 2, 24, 16, 40, 48, 2, 32, 24, 8, 2, 4, 2,
                             72, 104, 160)),
}


def get_pokepel_config(name: str, **overrides) -> PokepelConfig:
    return dataclasses.replace(POKEPEL_CONFIGS[name], **overrides)


class PokepelLayer(nn.Module):
    def __init__(self, config: PokepelConfig, layer: dict):
        super().__init__()
        width = config.hidden_size
        mlp = layer.get("mlp")
        for kind, known in ((layer["type"], MIXERS),
                            ((mlp or {}).get("kind", "dense"), MLPS)):
            if kind not in known:
                raise ValueError(f"unknown layer kind {kind!r}; this model "
                                 f"has {sorted(known)}")
        self.eps = config.norm_eps
        self.norm1 = nn.Parameter(torch.ones(width))
        self.block = GatedParallel(
            width, MIXERS[layer["type"]](width, layer["mixer"], self.eps),
            mlp and MLPS[mlp.get("kind", "dense")](width, mlp, self.eps))

    def cache_specs(self):
        return self.block.cache_specs()

    def load(self, get, prefix):
        copy_weight(self.norm1, get(prefix + "norm1"))
        self.block.load(get, prefix)

    def forward(self, x, pending, batch, pools):
        """(x, pending) -> (x, pending): the stream is x + pending; the gates,
        the residual add and the next norm are one kernel."""
        x, h, _ = sv.residual_norm(x, pending, self.eps, self.norm1)
        return x, self.block(h, batch, pools)


class PokepelForCausalLM(nn.Module):
    """Served through ``inference.InferenceEngine`` (``forward_ragged``)."""
    supports_ragged = True

    def __init__(self, config: PokepelConfig):
        super().__init__()
        if ps.get_tensor_model_parallel_size() != 1:
            raise NotImplementedError(
                "Pokepel is served one model per GPU (all heads of an "
                "attention share one latent); tensor parallelism is not "
                "implemented")
        W, V = config.hidden_size, config.vocab_size
        self.config = config
        self.embed = ParallelEmbedding(V, W)
        self.layers = nn.ModuleList(PokepelLayer(config, l)
                                    for l in config.layers)
        self.final_norm = nn.Parameter(torch.ones(W))
        self.head = nn.Parameter(torch.randn(V, W) * W ** -0.5)

    def load_checkpoint(self, tensors: dict):
        """Fill every parameter from a name -> tensor dictionary; a missing,
        unused or misshapen tensor is an error."""
        get = CheckpointReader(tensors)
        copy_weight(self.embed.weight, get("embed"))
        for i, layer in enumerate(self.layers):
            layer.load(get, f"l{i}.")
        copy_weight(self.final_norm, get("final.norm"))
        copy_weight(self.head, get("head"))
        get.done()

    def cache_specs(self):
        return [layer.cache_specs() for layer in self.layers]

    def forward_ragged(self, batch, pools):
        """Packed step -> float32 logits (wanted, vocab), or None."""
        x, pending = None, sv.Pending(self.embed(batch.tokens))
        for layer, pool in zip(self.layers, pools):
            x, pending = layer(x, pending, batch, pool)
        if not batch.want.shape[0]:
            return None
        _, h, _ = sv.residual_norm(x, pending, self.config.norm_eps,
                                   self.final_norm, keep_x=False,
                                   index=batch.want)
        return sv.linear_f32(h, self.head)

    def forward(self, *args, **kwargs):
        raise NotImplementedError("Pokepel runs through the serving engine: "
                                  "inference.generate or InferenceEngine")
