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
from typing import List, Optional, Sequence

import torch
import torch.nn as nn

from ..inference.paged_cache import (ConvRing, MatrixState, PagedKV,
                                     PagedLatent)
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

    def skip(self, name: str):
        """This tensor may be there, and has no place."""
        self.used.add(name)

    def done(self):
        extra = set(self.tensors) - self.used
        if extra:
            raise KeyError(f"checkpoint tensors without a place: "
                           f"{sorted(extra)[:5]}")


class Projected(nn.Module):
    """What reads projections of the layer's rows that one product makes.
    ``names`` are the checkpoint names of the projections in the order in
    which they are stacked, ``sizes`` their widths."""
    names: Sequence[str] = ()
    sizes: Sequence[int] = ()
    padding = 0         # rows of zeros behind the projections

    def stacked(self, get, prefix) -> Optional[torch.Tensor]:
        parts = [get(prefix + n) for n in self.names]
        for p, n, s in zip(parts, self.names, self.sizes):
            if p.shape[0] != s:
                raise ValueError(f"{prefix}{n} has {p.shape[0]} rows, "
                                 f"expected {s}")
        if not parts:
            return None
        if self.padding:
            parts.append(parts[0].new_zeros(self.padding, parts[0].shape[1]))
        return torch.cat(parts)

    def split(self, proj):
        out, at = [], 0
        for s in self.sizes:
            out.append(proj[:, at:at + s])
            at += s
        return out


class Mixer(Projected):
    """Mixes the rows of a request; keeps something between steps."""

    def cache_specs(self) -> list:
        raise NotImplementedError


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


class ScoredAttention(Mixer):
    """Causal softmax attention with grouped key/value heads and modified
    scores; what is None or zero is left out.

    rot        rotation of neighbouring pairs: base, dims, scaling
    qk_norm    RMS norm of queries and keys, a head: "plain" or "weighted"
    q_temp     queries grow with their position: coef, every
    slopes     distance bias, a number a head
    head_temp  a learned factor of the scores, a head
    softcap    cap of the scores
    sink       a score of the denominator alone: "zero" or "learned"
    gate       a sigmoid gate a head
    v_mix      values take a share of those of the first layer that has it
    """

    def __init__(self, width, heads, kv_heads, dim, vdim, scale, eps,
                 rot=None, qk_norm=None, q_temp=None, slopes=None,
                 head_temp=False, softcap=0.0, sink=None, gate=False,
                 v_mix=False):
        super().__init__()
        if heads % kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        if rot and (rot["dims"] % 2 or not 0 <= rot["dims"] <= dim):
            raise ValueError(f"{rot['dims']} of {dim} dimensions turn")
        if qk_norm not in (None, "plain", "weighted") or \
                sink not in (None, "zero", "learned"):
            raise ValueError(f"norm {qk_norm!r}, sink {sink!r}")
        if slopes is not None and len(slopes) != heads:
            raise ValueError("one slope per head")
        if max(dim, vdim) > sv.MAX_HEAD_DIM:
            raise ValueError(f"head size {max(dim, vdim)} > "
                             f"{sv.MAX_HEAD_DIM}")
        self.heads, self.scale, self.eps = heads, scale, eps
        self.rot, self.qk_norm = rot, qk_norm
        self.q_temp = (q_temp["coef"], int(q_temp["every"])) if q_temp \
            else (0.0, 0)
        self.slopes, self.softcap = slopes, softcap or 0.0
        self.v_mix, self.gated = v_mix, gate
        self.kv = PagedKV(kv_heads, dim, vdim)
        self.names = ("q", "k", "v") + (("g",) if gate else ())
        self.sizes = (heads * dim, kv_heads * dim, kv_heads * vdim) + \
            ((heads,) if gate else ())
        # a whole number of 16-byte words a row
        self.padding = -sum(self.sizes) % 8
        self.loads = []
        if qk_norm == "weighted":
            self.q_norm, self.k_norm = _vector(dim), _vector(dim)
            self.loads += [("q_norm", "q.norm"), ("k_norm", "k.norm")]
        if head_temp:
            self.temp = _vector(heads)
            self.loads.append(("temp", "temp"))
        if sink == "learned":
            self.sink = nn.Parameter(torch.zeros(heads))
            self.loads.append(("sink", "sink"))
        elif sink == "zero":
            self.register_buffer("sink", torch.zeros(heads),
                                 persistent=False)
        if v_mix:
            self.mix = nn.Parameter(torch.full((), 0.5))
            self.loads.append(("mix", "vmix"))
        self.o = _row(heads * vdim, width)
        self._const = None

    def cache_specs(self):
        return [self.kv]

    def load(self, get, prefix):
        for name, key in self.loads:
            copy_weight(getattr(self, name), get(prefix + key))
        if not self.v_mix:
            get.skip(prefix + "vmix")
        copy_weight(self.o.weight, get(prefix + "o"))

    def _constants(self, device):
        if self._const is None or self._const[0] != device:
            freq = sv.rotary_frequencies(
                self.rot["base"], self.rot["dims"], device,
                self.rot.get("scaling")) if self.rot else None
            slope = None if self.slopes is None else torch.tensor(
                self.slopes, dtype=torch.float64).float().to(device)
            self._const = device, freq, slope
        return self._const[1:]

    def forward(self, h, proj, batch, pools, values: Optional[list] = None):
        """``values`` is a step's list of the values that layers share: the
        first layer that mixes puts its own there."""
        q, k, v, *g = self.split(proj)
        freq, slope = self._constants(h.device)
        prep = sv.QkvPrep(freq=freq, norm=self.qk_norm is not None,
                          q_norm=getattr(self, "q_norm", None),
                          k_norm=getattr(self, "k_norm", None), eps=self.eps,
                          temp_coef=self.q_temp[0], temp_every=self.q_temp[1])
        if self.v_mix:
            if values:
                prep.first, prep.mix = values[0], self.mix
            else:
                values.append(v)
        mod = sv.ScoreMod(temp=getattr(self, "temp", None), cap=self.softcap,
                          slope=slope, sink=getattr(self, "sink", None),
                          gate=g[0] if g else None)
        return self.o(sv.ragged_attention(q, k, v, batch, pools[0],
                                          self.heads, self.scale, prep=prep,
                                          mod=mod))


def alibi_slopes(heads: int) -> List[float]:
    return [2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)]


def rotation(base, dims, scaling, device):
    """Frequencies, scaled as YaRN does or plain, and their amplitude."""
    if scaling:
        return sv.yarn_frequencies(base, dims, device, scaling)
    return sv.rotary_frequencies(base, dims, device), 1.0


class LatentAttention(Mixer):
    """Softmax attention whose keys and values are projections of a small
    latent, which alone is cached beside one rotated key part that all heads
    share; a sliding window (0: plain causal) and a sigmoid gate on the
    heads.  Every query head is [unrotated | rotated].

    pairs      neighbours turn together, not element i and i + rot_dims / 2
    scaling    of the rotation, see ``serving.yarn_frequencies``
    sink       a learned score a head joins the denominator
    """
    names = ("q", "dkv", "g")

    def __init__(self, width, heads, dim, rot_dim, vdim, rank, scale,
                 rot_base, rot_dims, eps, window=0, pairs=False, scaling=None,
                 sink=False):
        super().__init__()
        if rot_dims % 2 or not 0 <= rot_dims <= rot_dim:
            raise ValueError(f"{rot_dims} of {rot_dim} dimensions turn")
        if rank + rot_dim > sv.MAX_LATENT_ROW:
            raise ValueError(f"latent row of {rank + rot_dim} > "
                             f"{sv.MAX_LATENT_ROW}")
        self.heads, self.dim, self.vdim = heads, dim, vdim
        self.rank, self.scale, self.eps = rank, scale, eps
        self.rot_base, self.rot_dims = rot_base, rot_dims
        self.pairs, self.scaling = pairs, scaling
        self.window = window
        self.latent = PagedLatent(rank, rot_dim, window)
        self.sizes = (heads * (dim + rot_dim), rank + rot_dim, heads * vdim)
        self.norm = _vector(rank)
        # W_uk twice: transposed per head for queries, with W_uv for keys
        self.absorb = nn.Parameter(
            torch.randn(heads, rank, dim) * rank ** -0.5)
        self.expand = nn.Parameter(
            torch.randn(heads * (dim + vdim), rank) * rank ** -0.5)
        self.sink = nn.Parameter(torch.zeros(heads)) if sink else None
        self._turn = None
        self.o = _row(heads * vdim, width)

    def cache_specs(self):
        return [self.latent]

    def load(self, get, prefix):
        uk = get(prefix + "uk")
        copy_weight(self.norm, get(prefix + "dkv.norm"))
        copy_weight(self.expand, torch.cat([uk, get(prefix + "uv")]))
        copy_weight(self.absorb, uk.view(self.heads, self.dim, self.rank)
                    .transpose(1, 2))
        if self.sink is not None:
            copy_weight(self.sink, get(prefix + "sink"))
        copy_weight(self.o.weight, get(prefix + "o"))

    def forward(self, h, proj, batch, pools):
        q, kv, g = self.split(proj)
        if self._turn is None or self._turn[0].device != h.device:
            self._turn = rotation(self.rot_base, self.rot_dims, self.scaling,
                                  h.device)
        w = sv.LatentWeights(self.norm, self.absorb, self.expand, *self._turn,
                             self.pairs, self.sink)
        return self.o(sv.latent_attention(
            q, kv, g, batch, pools[0], w, self.heads, self.dim, self.vdim,
            self.scale, self.eps, self.window))


class _MatrixMemory(Mixer):
    """A recurrent matrix state per head, a group-normed and gated output."""
    names = ("q", "k", "v", "g")
    normalized = False
    weighted = True       # the norm
    silu_gate = False     # instead of a sigmoid

    def __init__(self, width, heads, dim, vdim, eps, norm_group):
        super().__init__()
        self.heads, self.dim, self.vdim, self.eps = heads, dim, vdim, eps
        self.norm_group = norm_group
        self.state = MatrixState(heads, dim, vdim, self.normalized)
        self.sizes = (heads * dim, heads * dim, heads * vdim, heads * vdim)
        self.norm = _vector(heads * vdim) if self.weighted else None
        self.o = _row(heads * vdim, width)

    def cache_specs(self):
        return [self.state]

    def load(self, get, prefix):
        if self.weighted:
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
                                    self.eps, self.silu_gate))


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


class Retention(_MatrixMemory):
    """Linear attention with a fixed decay per head on rotated queries and keys
    (element i turns with i + dims / 2; keys times dim^-1/2); every head is
    normed on its own, without a weight, and gated by silu."""
    weighted, silu_gate = False, True

    def __init__(self, width, heads, dim, vdim, decay, eps, rot_base,
                 rot_dims, scaling=None):
        super().__init__(width, heads, dim, vdim, eps, norm_group=vdim)
        if len(decay) != heads:
            raise ValueError("one decay per head")
        if rot_dims % 2 or not 0 <= rot_dims <= dim:
            raise ValueError(f"{rot_dims} of {dim} dimensions turn")
        if dim > sv.MAX_HEAD_DIM:
            raise ValueError(f"key size {dim} > {sv.MAX_HEAD_DIM}")
        self.decay = [float(d) for d in decay]
        self.rot = rot_base, rot_dims, scaling
        self._gate = None

    def gate(self, h):
        if self._gate is None or self._gate.decay.device != h.device:
            d = sv.decay_gate(self.decay, h.device)
            self._gate = sv.TurnGate(d.decay, d.log2_decay, self.dim ** -0.5,
                                     *rotation(*self.rot, h.device))
        return self._gate

    def forward(self, h, proj, batch, pools):
        q, k, v, g = self.split(proj)
        S, gate = pools[0][0], self.gate(h)
        n, T = batch.portion_tokens, h.shape[0]
        out = torch.empty(T, self.heads * self.vdim, dtype=h.dtype,
                          device=h.device)
        done = 0          # rows that are normed and gated
        if n:
            if gate.norm_fits(h.dtype, self.dim, self.vdim, q, k, v, g):
                done = n
            sv.memory_mix(q[:n], k[:n], v[:n], gate, S, None, None,
                          batch.portions, self.heads, batch.chunks,
                          batch.chunk_first, out=out[:n],
                          silu_gate=g[:n] if done else None, eps=self.eps)
        if n < T:
            sv.memory_mix(q, k, v, gate, S, None, None, batch.singles,
                          self.heads, out=out)
        if done < T:
            sv.gated_norm(out[done:], None, g[done:], self.vdim, self.eps,
                          True, out=out[done:])
        return self.o(out)


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


class StateSpaceMemory(Mixer):
    """State-space duality (Mamba-2): a matrix state per head whose decay and
    input weight come from a projected time step; x, B and C pass a short causal
    convolution and silu, heads share B and C in groups; a skip of x, a silu
    gate, then a norm over ``norm_groups`` equal parts."""
    names = ("in",)

    def __init__(self, width, heads, vdim, state, groups, taps, norm_groups,
                 eps):
        super().__init__()
        inner = heads * vdim
        if heads % groups or inner % norm_groups:
            raise ValueError(f"{heads} heads in {groups} groups, {inner} "
                             f"columns in {norm_groups}")
        if state > sv.MAX_HEAD_DIM or not 1 <= taps <= sv.MAX_TAPS:
            raise ValueError(f"state of {state}, {taps} taps")
        self.heads, self.eps, self.norm_group = heads, eps, \
            inner // norm_groups
        self.parts = (inner, groups * state, groups * state)   # x, B, C
        channels = sum(self.parts)
        self.sizes = (inner, channels)
        self.padding = -sum(self.sizes) % 8
        self.memory = MatrixState(heads, state, vdim)
        self.ring = ConvRing(channels, taps)
        self.step_proj = nn.Parameter(
            torch.randn(heads, width) * width ** -0.5)
        self.step_bias = nn.Parameter(torch.zeros(heads))
        self.A_log = nn.Parameter(torch.zeros(heads))
        self.skip = _vector(heads)
        self.conv = nn.Parameter(torch.full((taps, channels), 1.0 / taps))
        self.conv_bias = nn.Parameter(torch.zeros(channels))
        self.norm = _vector(inner)
        self.o = _row(inner, width)

    def cache_specs(self):
        return [self.memory, self.ring]

    def stacked(self, get, prefix):
        w = get(prefix + "in")
        n = sum(self.sizes)
        if w.shape[0] != n + self.heads:
            raise ValueError(f"{prefix}in has {w.shape[0]} rows, expected "
                             f"{n + self.heads}")
        return torch.cat([w[:n], w.new_zeros(self.padding, w.shape[1])])

    def load(self, get, prefix):
        copy_weight(self.step_proj, get(prefix + "in")[-self.heads:])
        copy_weight(self.conv, get(prefix + "conv").t())
        for name, key in (("step_bias", "dt_bias"), ("A_log", "A_log"),
                          ("skip", "D"), ("conv_bias", "conv.b"),
                          ("norm", "norm")):
            copy_weight(getattr(self, name), get(prefix + key))
        copy_weight(self.o.weight, get(prefix + "o"))

    def forward(self, h, proj, batch, pools):
        (S, _, _), ring = pools
        z, xbc = self.split(proj)
        step = sv.linear_f32(h, self.step_proj)
        conv = sv.ShortConv(self.conv, ring, self.conv_bias)
        n, T = batch.portion_tokens, h.shape[0]
        out = torch.empty_like(z, memory_format=torch.contiguous_format)

        def mix(a, b, x, seg, **kw):
            v, k, q = x.split(self.parts, dim=1)
            gate = sv.TimeGate(step[a:b], self.step_bias, self.A_log,
                               self.skip, z[a:b], kw.pop("conv", None))
            sv.memory_mix(q, k, v, gate, S, None, None, seg, self.heads,
                          out=out[a:b], **kw)

        if n:
            x = sv.short_conv(xbc[:n], conv, batch.portions, batch.chunks,
                              silu=True)
            mix(0, n, x, batch.portions, chunks=batch.chunks,
                chunk_first=batch.chunk_first)
        if n < T:      # the rows of a segment count from the whole batch
            mix(0, T, xbc, batch.singles, conv=conv)
        return self.o(sv.gated_norm(out, self.norm, None, self.norm_group,
                                    self.eps))


class SingleMixer(nn.Module):
    """One mixer with its projection."""

    def __init__(self, width, mixer: Mixer):
        super().__init__()
        self.mixer = mixer
        self.proj = _column(width, sum(mixer.sizes) + mixer.padding)

    def cache_specs(self) -> List:
        return self.mixer.cache_specs()

    def load(self, get, prefix):
        copy_weight(self.proj.weight, self.mixer.stacked(get, prefix))
        self.mixer.load(get, prefix)

    def forward(self, h, batch, pools, **shared) -> sv.Pending:
        return sv.Pending(self.mixer(h, self.proj(h), batch, pools,
                                     **shared))


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


_side_streams = {}


def side_stream(device) -> torch.cuda.Stream:
    """A second stream of the device, for work beside the current one's."""
    if device not in _side_streams:
        _side_streams[device] = torch.cuda.Stream(device)
    return _side_streams[device]


class GatedParallel(nn.Module):
    """A mixer and a feed-forward (or none) side by side on the same rows h,
    each result times sigmoid(W h + b) of its own.  One product makes the
    projections of both and the gates; the results are left pending.

    In steps of single tokens, what the feed-forward can do ``ahead`` of the
    projections runs on a second stream (a second branch of a captured graph),
    beside the mixer's small kernels."""

    def __init__(self, width, mixer: Mixer, mlp: Optional[Projected] = None):
        super().__init__()
        self.mixer, self.mlp = mixer, mlp
        self.bias1 = nn.Parameter(torch.zeros(width))
        if mlp is not None:
            self.bias2 = nn.Parameter(torch.zeros(width))
        sizes = [sum(mixer.sizes) + mixer.padding, width]
        if mlp is not None:
            sizes += [sum(mlp.sizes) + mlp.padding, width]
        # every part starts at a 16-byte word
        self.at, n = [], 0
        for s in sizes:
            self.at.append((n, n + s))
            n += s + -s % 8
        self.proj = _column(width, n)

    def cache_specs(self) -> List:
        return self.mixer.cache_specs()

    def load(self, get, prefix):
        w = torch.zeros_like(self.proj.weight)
        parts = [self.mixer.stacked(get, prefix + "mix."),
                 get(prefix + "rg1")]
        copy_weight(self.bias1, get(prefix + "rg1.b"))
        self.mixer.load(get, prefix + "mix.")
        if self.mlp is not None:
            parts += [self.mlp.stacked(get, prefix + "mlp."),
                      get(prefix + "rg2")]
            copy_weight(self.bias2, get(prefix + "rg2.b"))
            self.mlp.load(get, prefix + "mlp.")
        else:
            get.skip(prefix + "rg2")
            get.skip(prefix + "rg2.b")
        for (a, b), part in zip(self.at, parts):
            if part is not None:
                copy_weight(w[a:b], part)
        copy_weight(self.proj.weight, w)

    def forward(self, h, batch, pools) -> sv.Pending:
        ahead = None
        beside = getattr(self.mlp, "ahead", None)
        here = torch.cuda.current_stream(h.device)
        if beside and not batch.portion_tokens:
            # what is allocated on either stream is used on the other only
            # between these two waits, or before the next layer's first
            side = side_stream(h.device)
            side.wait_stream(here)
            with torch.cuda.stream(side):
                ahead = beside(h)
        proj = self.proj(h)
        mix, gate1, *rest = [proj[:, a:b] for a, b in self.at]
        branches = [sv.Branch(self.mixer(h, mix, batch, pools), gate=gate1,
                              bias=self.bias1)]
        if self.mlp is not None:
            y = self.mlp(h, rest[0], ahead)
            y.gate, y.bias = rest[1], self.bias2
            branches.append(y)
        if ahead is not None:
            here.wait_stream(side)
        return sv.Pending(branches=branches)


class PolyNormMLP(Projected):
    """down(a N(z) + b N(z^2) + c N(z^3) + e) of z = up h, where powers are
    taken element by element and N divides a row by its root mean square."""
    names = ("up",)

    def __init__(self, width, ff, eps):
        super().__init__()
        self.sizes, self.eps = (ff,), eps
        self.act = nn.Parameter(torch.tensor([1.0, 0.0, 0.0, 0.0]))
        self.down = _row(ff, width)

    def load(self, get, prefix):
        copy_weight(self.act, get(prefix + "act"))
        copy_weight(self.down.weight, get(prefix + "down"))

    def forward(self, h, proj, ahead=None) -> sv.Branch:
        return sv.Branch(self.down(sv.poly_norm(self.split(proj)[0], self.act,
                                                self.eps)))


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
    """A router with a bias (``bias_name`` None: without) and gated experts:
    min(g, limit) sigmoid(alpha g) (clamp(u, limit) + shift); the chosen experts
    are summed, weighted as ``routing`` (or the plain routing, if it is a number
    of experts) says.  The sum is left pending, so it fuses into the next
    residual norm."""

    def __init__(self, width, ff, experts, routing, limit=math.inf, alpha=1.0,
                 shift=0.0, bias_name: Optional[str] = "router.b"):
        super().__init__()
        self.routing = sv.Routing(routing) if isinstance(routing, int) \
            else routing
        self.routing.check(experts)
        self.act, self.bias_name = (alpha, limit, shift), bias_name
        self.router = nn.Parameter(
            torch.randn(experts, width) * width ** -0.5)
        self.bias = nn.Parameter(torch.zeros(experts)) if bias_name else None
        self.gate_up = nn.Parameter(torch.empty(experts, 2 * ff, width))
        self.down = nn.Parameter(torch.empty(experts, width, ff))
        nn.init.normal_(self.gate_up, std=width ** -0.5)
        nn.init.normal_(self.down, std=ff ** -0.5)

    def load(self, get, prefix):
        copy_weight(self.router, get(prefix + "router"))
        if self.bias is not None:
            copy_weight(self.bias, get(prefix + self.bias_name))
        for e, (gu, down) in enumerate(zip(self.gate_up, self.down)):
            p = f"{prefix}e{e}."
            copy_weight(gu, torch.cat([get(p + "gate"), get(p + "up")]))
            copy_weight(down, get(p + "down"))

    def forward(self, h) -> sv.Pending:
        return sv.moe_mlp(h, sv.linear_f32(h, self.router), self.bias,
                          self.gate_up, self.down, self.routing, *self.act)


class SharedExpertsMLP(Projected):
    """Experts beside one (of ``shared_ff``, 0: none) that every row uses, whose
    projections come with the layer's."""

    def __init__(self, width, experts: ExpertsMLP, shared_ff=0):
        super().__init__()
        self.experts = experts
        if shared_ff:
            self.names = ("shared.gate", "shared.up")
            self.sizes = (shared_ff, shared_ff)
            self.down = _row(shared_ff, width)

    def load(self, get, prefix):
        self.experts.load(get, prefix)
        if self.sizes:
            copy_weight(self.down.weight, get(prefix + "shared.down"))

    def ahead(self, h) -> sv.Pending:
        return self.experts(h)

    def forward(self, h, proj, ahead=None) -> sv.Branch:
        y = ahead or self.experts(h)
        plus = self.down(sv.silu_mul(proj)) if self.sizes else None
        return sv.Branch(y.delta, y.coef, plus)


class TokenSide(nn.Module):
    """A vector of the token, of this layer's columns of a table, gated by the
    stream: proj(gelu(gate x) * table[token]), normed on its way into the
    stream.  The table belongs to the model."""

    def __init__(self, width, dim, layer):
        super().__init__()
        self.at = layer * dim
        self.gate, self.proj = _column(width, dim), _row(dim, width)
        self.norm = _vector(width)

    def load(self, get, prefix):
        copy_weight(self.gate.weight, get(prefix + "gate"))
        copy_weight(self.proj.weight, get(prefix + "proj"))
        copy_weight(self.norm, get(prefix + "norm"))

    def forward(self, x, table, tokens) -> sv.Pending:
        g = sv.gelu_rows_(self.gate(x), table, tokens, self.at)
        return sv.Pending(self.proj(g), w1=self.norm)
