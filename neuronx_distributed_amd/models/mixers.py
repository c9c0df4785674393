"""Token mixers and feed-forwards for ragged serving batches.

Building blocks that a decoder design composes; every size and constant is a
parameter.  A mixer reads the normed rows h (T, width) of a packed batch and
its own cache pools, and returns the pending residual update.  Portions of
prompts occupy the first rows, single tokens the rest; each kind runs its
own kernels into one output.

The projections of a mixer are ONE column-parallel GEMM whose output the
kernels read as strided slices.
"""

import math
from typing import List, Sequence

import torch
import torch.nn as nn

from ..inference.paged_cache import MatrixState, PagedKV, PagedLatent
from ..ops import serving as sv
from ..parallel.layers import ColumnParallelLinear, RowParallelLinear


def _column(width, out):
    return ColumnParallelLinear(width, out, bias=False, gather_output=False)


def _row(inp, width):
    return RowParallelLinear(inp, width, bias=False, input_is_parallel=True)


def _vector(n):
    return nn.Parameter(torch.ones(n))


def copy_weight(param: torch.Tensor, value: torch.Tensor):
    if param.shape != value.shape:
        raise ValueError(f"weight of shape {tuple(value.shape)}, expected "
                         f"{tuple(param.shape)}")
    with torch.no_grad():
        param.copy_(value)


class CheckpointReader:
    """Hands out the tensors of a name -> tensor dictionary; a missing or
    (``done``) an unused one is an error."""

    def __init__(self, tensors: dict):
        self.tensors, self.used = tensors, set()

    def __call__(self, name: str) -> torch.Tensor:
        if name not in self.tensors:
            raise KeyError(f"checkpoint has no tensor {name!r}")
        self.used.add(name)
        return self.tensors[name]

    def done(self):
        extra = set(self.tensors) - self.used
        if extra:
            raise KeyError(f"checkpoint tensors without a place: "
                           f"{sorted(extra)[:5]}")


class Mixer(nn.Module):
    """``names`` are the checkpoint names of the projections in the order in
    which they are stacked, ``sizes`` their widths."""
    names: Sequence[str]
    sizes: Sequence[int]

    def cache_specs(self) -> list:
        raise NotImplementedError

    def stacked(self, get, prefix) -> torch.Tensor:
        parts = [get(prefix + n) for n in self.names]
        for p, n, s in zip(parts, self.names, self.sizes):
            if p.shape[0] != s:
                raise ValueError(f"{prefix}{n} has {p.shape[0]} rows, "
                                 f"expected {s}")
        return torch.cat(parts)

    def split(self, proj):
        out, at = [], 0
        for s in self.sizes:
            out.append(proj[:, at:at + s])
            at += s
        return out


class SlidingAttention(Mixer):
    """Softmax attention without rotation: grouped key/value heads, unequal
    query/key and value sizes, a sliding window that keeps the first tokens
    visible (window 0: plain causal)."""
    names = ("q", "k", "v")

    def __init__(self, width, heads, kv_heads, dim, vdim, scale, window=0,
                 keep_first=0):
        super().__init__()
        if heads % kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        self.heads, self.scale = heads, scale
        self.window, self.keep_first = window, keep_first
        self.kv = PagedKV(kv_heads, dim, vdim, window, keep_first)
        self.sizes = (heads * dim, kv_heads * dim, kv_heads * vdim)
        self.out_size = heads * vdim
        self.o = _row(self.out_size, width)

    def cache_specs(self):
        return [self.kv]

    def load(self, get, prefix):
        copy_weight(self.o.weight, get(prefix + "o"))

    def forward(self, h, proj, batch, pools):
        q, k, v = self.split(proj)
        return self.o(sv.ragged_attention(
            q, k, v, batch, pools[0], self.heads, self.scale, self.window,
            self.keep_first))


class LatentAttention(Mixer):
    """Softmax attention whose keys and values are projections of a small
    latent, which alone is cached beside one rotated key part that all heads
    share; a sliding window (0: plain causal) and a sigmoid gate on the
    heads.  Every query head is [unrotated | rotated]."""
    names = ("q", "dkv", "g")

    def __init__(self, width, heads, dim, rot_dim, vdim, rank, scale,
                 rot_base, rot_dims, eps, window=0):
        super().__init__()
        if rot_dims % 2 or not 0 <= rot_dims <= rot_dim:
            raise ValueError(f"{rot_dims} of {rot_dim} dimensions turn")
        if rank + rot_dim > sv.MAX_LATENT_ROW:
            raise ValueError(f"latent row of {rank + rot_dim} > "
                             f"{sv.MAX_LATENT_ROW}")
        self.heads, self.dim, self.vdim = heads, dim, vdim
        self.rank, self.scale, self.eps = rank, scale, eps
        self.rot_base, self.rot_dims = rot_base, rot_dims
        self.window = window
        self.latent = PagedLatent(rank, rot_dim, window)
        self.sizes = (heads * (dim + rot_dim), rank + rot_dim, heads * vdim)
        self.norm = _vector(rank)
        # W_uk twice: transposed per head for queries, with W_uv for keys
        self.absorb = nn.Parameter(
            torch.randn(heads, rank, dim) * rank ** -0.5)
        self.expand = nn.Parameter(
            torch.randn(heads * (dim + vdim), rank) * rank ** -0.5)
        self._freq = None
        self.o = _row(heads * vdim, width)

    def cache_specs(self):
        return [self.latent]

    def load(self, get, prefix):
        uk = get(prefix + "uk")
        copy_weight(self.norm, get(prefix + "dkv.norm"))
        copy_weight(self.expand, torch.cat([uk, get(prefix + "uv")]))
        copy_weight(self.absorb, uk.view(self.heads, self.dim, self.rank)
                    .transpose(1, 2))
        copy_weight(self.o.weight, get(prefix + "o"))

    def forward(self, h, proj, batch, pools):
        q, kv, g = self.split(proj)
        if self._freq is None or self._freq.device != h.device:
            self._freq = sv.rotary_frequencies(self.rot_base, self.rot_dims,
                                               h.device)
        w = sv.LatentWeights(self.norm, self.absorb, self.expand, self._freq)
        return self.o(sv.latent_attention(
            q, kv, g, batch, pools[0], w, self.heads, self.dim, self.vdim,
            self.scale, self.eps, self.window))


class _MatrixMemory(Mixer):
    """A recurrent matrix state per head, a group-normed and gated output."""
    names = ("q", "k", "v", "g")
    normalized = False

    def __init__(self, width, heads, dim, vdim, eps, norm_group):
        super().__init__()
        self.heads, self.dim, self.vdim, self.eps = heads, dim, vdim, eps
        self.norm_group = norm_group
        self.state = MatrixState(heads, dim, vdim, self.normalized)
        self.sizes = (heads * dim, heads * dim, heads * vdim, heads * vdim)
        self.norm = _vector(heads * vdim)
        self.o = _row(heads * vdim, width)

    def cache_specs(self):
        return [self.state]

    def load(self, get, prefix):
        copy_weight(self.norm, get(prefix + "norm"))
        copy_weight(self.o.weight, get(prefix + "o"))

    def gate(self, h):
        raise NotImplementedError

    def forward(self, h, proj, batch, pools):
        q, k, v, g = self.split(proj)
        S, n, m = pools[0]
        gate = self.gate(h)
        out = torch.empty(h.shape[0], self.heads * self.vdim, dtype=h.dtype,
                          device=h.device)
        if batch.portions.shape[0]:
            sv.memory_mix(q, k, v, gate, S, n, m, batch.portions, self.heads,
                          batch.chunks, batch.chunk_first, out=out)
        if batch.singles.shape[0]:
            sv.memory_mix(q, k, v, gate, S, n, m, batch.singles, self.heads,
                          out=out)
        return self.o(sv.gated_norm(out, self.norm, g, self.norm_group,
                                    self.eps))


class DecayMemory(_MatrixMemory):
    """Lightning attention: a fixed decay per head, silu on q, k and v, one
    norm over all heads."""

    def __init__(self, width, heads, dim, vdim, decay, eps):
        super().__init__(width, heads, dim, vdim, eps,
                         norm_group=heads * vdim)
        if len(decay) != heads:
            raise ValueError("one decay per head")
        self.decay = [float(d) for d in decay]
        self._gate = None

    def gate(self, h):
        if self._gate is None or self._gate.decay.device != h.device:
            self._gate = sv.decay_gate(self.decay, h.device)
        return self._gate


class GatedMemory(_MatrixMemory):
    """Exponentially gated matrix memory with a normaliser and a running
    maximum; every head is normed on its own."""
    normalized = True

    def __init__(self, width, heads, dim, vdim, gate_cap, eps):
        super().__init__(width, heads, dim, vdim, eps, norm_group=vdim)
        self.gate_cap = gate_cap
        self.gate_proj = nn.Parameter(torch.zeros(2 * heads, width))
        self.i_bias = nn.Parameter(torch.zeros(heads))
        self.f_bias = nn.Parameter(torch.zeros(heads))

    def load(self, get, prefix):
        super().load(get, prefix)
        copy_weight(self.gate_proj, torch.cat([get(prefix + "i"),
                                               get(prefix + "f")]))
        copy_weight(self.i_bias, get(prefix + "i.b"))
        copy_weight(self.f_bias, get(prefix + "f.b"))

    def gate(self, h):
        return sv.ExpGate(sv.linear_f32(h, self.gate_proj), self.i_bias,
                          self.f_bias, self.gate_cap,
                          1.0 / math.sqrt(self.dim))


class SingleMixer(nn.Module):
    """One mixer with its projection."""

    def __init__(self, width, mixer: Mixer):
        super().__init__()
        self.mixer = mixer
        self.proj = _column(width, sum(mixer.sizes))

    def cache_specs(self) -> List:
        return self.mixer.cache_specs()

    def load(self, get, prefix):
        copy_weight(self.proj.weight, self.mixer.stacked(get, prefix))
        self.mixer.load(get, prefix)

    def forward(self, h, batch, pools) -> sv.Pending:
        return sv.Pending(self.mixer(h, self.proj(h), batch, pools))


class ParallelMixer(nn.Module):
    """Two mixers side by side on the same rows, one projection GEMM for
    both.  The result is ``branch_scale`` times the sum of the two outputs,
    each RMS-normed over the width with its own weight; that sum is left
    pending, so it fuses into the next residual norm."""

    def __init__(self, width, left: Mixer, right: Mixer,
                 branch_scale: float = 0.5):
        super().__init__()
        self.left, self.right = left, right
        self.branch_scale = branch_scale
        self.n_left = sum(left.sizes)
        self.proj = _column(width, self.n_left + sum(right.sizes))
        self.left_out, self.right_out = _vector(width), _vector(width)

    def cache_specs(self) -> List:
        return self.left.cache_specs() + self.right.cache_specs()

    def load(self, get, prefix):
        copy_weight(self.proj.weight, torch.cat([
            self.left.stacked(get, prefix + "left."),
            self.right.stacked(get, prefix + "right.")]))
        for name in ("left", "right"):
            getattr(self, name).load(get, f"{prefix}{name}.")
            copy_weight(getattr(self, name + "_out"),
                        get(f"{prefix}{name}.out"))

    def forward(self, h, batch, pools) -> sv.Pending:
        p = self.proj(h)
        n = len(self.left.cache_specs())
        return sv.Pending(
            self.left(h, p[:, :self.n_left], batch, pools[:n]),
            self.right(h, p[:, self.n_left:], batch, pools[n:]),
            self.left_out, self.right_out, self.branch_scale)


class _PlainMLP(nn.Module):
    """down(act(up x))"""
    act = None

    def __init__(self, width, ff):
        super().__init__()
        self.up, self.down = _column(width, ff), _row(ff, width)

    def load(self, get, prefix):
        copy_weight(self.up.weight, get(prefix + "up"))
        copy_weight(self.down.weight, get(prefix + "down"))

    def forward(self, h) -> sv.Pending:
        return sv.Pending(self.down(self.act(self.up(h))))


class ReluSquaredMLP(_PlainMLP):
    act = staticmethod(sv.relu_squared_)


class GeluMLP(_PlainMLP):
    """The tanh form of gelu."""
    act = staticmethod(sv.gelu_tanh_)


class ExpertsMLP(nn.Module):
    """A router with a bias and gated experts: min(g, limit) sigmoid(alpha g)
    (clamp(u, limit) + shift); the ``top`` experts with the largest logits
    are summed, weighted by a softmax over their logits.  The sum is left
    pending, so it fuses into the next residual norm."""

    def __init__(self, width, ff, experts, top, limit=math.inf, alpha=1.0,
                 shift=0.0):
        super().__init__()
        if experts > sv.MAX_EXPERTS or not 1 <= top <= min(experts, 64):
            raise ValueError(f"{top} of {experts} experts")
        self.top, self.act = top, (alpha, limit, shift)
        self.router = nn.Parameter(
            torch.randn(experts, width) * width ** -0.5)
        self.bias = nn.Parameter(torch.zeros(experts))
        self.gate_up = nn.Parameter(torch.empty(experts, 2 * ff, width))
        self.down = nn.Parameter(torch.empty(experts, width, ff))
        nn.init.normal_(self.gate_up, std=width ** -0.5)
        nn.init.normal_(self.down, std=ff ** -0.5)

    def load(self, get, prefix):
        copy_weight(self.router, get(prefix + "router"))
        copy_weight(self.bias, get(prefix + "router.b"))
        for e, (gu, down) in enumerate(zip(self.gate_up, self.down)):
            p = f"{prefix}e{e}."
            copy_weight(gu, torch.cat([get(p + "gate"), get(p + "up")]))
            copy_weight(down, get(p + "down"))

    def forward(self, h) -> sv.Pending:
        return sv.moe_mlp(h, sv.linear_f32(h, self.router), self.bias,
                          self.gate_up, self.down, self.top, *self.act)
