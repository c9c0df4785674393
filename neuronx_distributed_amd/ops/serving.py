"""Serving kernels: ragged batches over a paged KV cache and state slots.

Python wrappers of ``libnxd_serving.so`` (``csrc/serving/*.hip``).  They run
on the GPU only — there is no eager substitute, a CPU tensor or a missing
library raises.  Activations and weights are bfloat16, or float32 in the
32-bit mode; the residual stream, attention scores and weights, norms,
gates and recurrent state are 32-bit in both.
"""

import ctypes
import math
import os
from dataclasses import dataclass, replace
from typing import Optional, Sequence, Union

import torch

PAGE_SIZE = 64
MAX_HEAD_DIM = 512          # attention q/k and v size, recurrent q/k size
MAX_LATENT_ROW = 1024       # latents and shared key columns of a cached row
MAX_EXPERTS = 512
MAX_TAPS = 65               # of a short convolution
EXPAND_MIN_TOKENS = 32      # shorter portions attend in the latent space
CHUNK = 256                 # tokens of one chunk of a matrix memory

_LIB = None


def library():
    global _LIB
    if _LIB is None:
        from .build import SERVING_LIB

        if not os.path.exists(SERVING_LIB):
            raise RuntimeError(
                f"{SERVING_LIB} is not built — run "
                "python -m neuronx_distributed_amd.ops.build")
        _LIB = ctypes.CDLL(SERVING_LIB)
    return _LIB


def ensure_built():
    """Compile the serving library if it is missing or out of date (and
    nothing else)."""
    from .build import build_group

    build_group("serving", verbose=False)


def _stream():
    return ctypes.c_void_p(torch.cuda.current_stream().cuda_stream)


def _p(t: Optional[torch.Tensor]):
    return None if t is None else t.data_ptr()


def _f32(t: torch.Tensor) -> int:
    if not t.is_cuda:
        raise RuntimeError("serving kernels run on the GPU only")
    if t.dtype not in (torch.bfloat16, torch.float32):
        raise TypeError(f"serving kernels take bfloat16 or float32, "
                        f"not {t.dtype}")
    return int(t.dtype == torch.float32)


def _check(status: int, what: str):
    if status:
        raise RuntimeError(f"{what}: launch failed with status {status}")


def _fields(names, ctype):
    return [(n, ctype) for n in names.split()]


class _BranchArgs(ctypes.Structure):
    _fields_ = (_fields("delta coef plus gate", ctypes.c_void_p)
                + _fields("gst", ctypes.c_long)
                + _fields("bias", ctypes.c_void_p)
                + _fields("parts", ctypes.c_long))


class _ResidualNormArgs(ctypes.Structure):
    _fields_ = (_fields("x delta delta2 w1 w2 coef vec x_out h w cat x0 "
                        "index conv ring singles hc", ctypes.c_void_p)
                + _fields("rows_out W delta_f32 parts groups p_groups taps "
                          "conv_row", ctypes.c_int)
                + _fields("eps scale w_base p_base h_scale", ctypes.c_float)
                + _fields("branches", ctypes.c_int)
                + [("br", _BranchArgs * 2)])


class _ConvArgs(ctypes.Structure):
    _fields_ = (_fields("x", ctypes.c_void_p) + _fields("xst", ctypes.c_long)
                + _fields("w bias out", ctypes.c_void_p)
                + _fields("ost", ctypes.c_long)
                + _fields("ring seg chunks", ctypes.c_void_p)
                + _fields("n_chunks chunk C taps silu add", ctypes.c_int))


class _QkvArgs(ctypes.Structure):
    _fields_ = (_fields("q k v", ctypes.c_void_p)
                + _fields("qst kst vst", ctypes.c_long)
                + _fields("freq qw kw first", ctypes.c_void_p)
                + _fields("fst", ctypes.c_long)
                + _fields("mix kc vc pos seq bt", ctypes.c_void_p)
                + _fields("MB T H G D E rot norm temp_every", ctypes.c_int)
                + _fields("temp_coef eps", ctypes.c_float))


class _ScoreArgs(ctypes.Structure):
    _fields_ = (_fields("temp sink slope gate", ctypes.c_void_p)
                + _fields("gst", ctypes.c_long)
                + _fields("cap", ctypes.c_float))


class _RowsArgs(ctypes.Structure):
    _fields_ = (_fields("q k v", ctypes.c_void_p)
                + _fields("qst kst vst", ctypes.c_long)
                + _fields("kc vc", ctypes.c_void_p)
                + _fields("kcs vcs", ctypes.c_long)
                + _fields("pos seq bt part out", ctypes.c_void_p)
                + _fields("MB rows H G D E splits append window keep",
                          ctypes.c_int)
                + _fields("scale", ctypes.c_float) + [("mod", _ScoreArgs)])


class _TilesArgs(ctypes.Structure):
    _fields_ = (_fields("q", ctypes.c_void_p) + _fields("qst", ctypes.c_long)
                + _fields("kc vc kr", ctypes.c_void_p)
                + _fields("kpage khead krow vpage vhead vrow rrow",
                          ctypes.c_long)
                + _fields("gate", ctypes.c_void_p)
                + _fields("gst", ctypes.c_long)
                + _fields("tiles bt out", ctypes.c_void_p)
                + _fields("MB H G D E DS window keep", ctypes.c_int)
                + _fields("scale", ctypes.c_float) + [("mod", _ScoreArgs)])


class _LatentAppendArgs(ctypes.Structure):
    _fields_ = (_fields("q", ctypes.c_void_p)
                + _fields("qst qh", ctypes.c_long)
                + _fields("qr", ctypes.c_void_p)
                + _fields("qrst qrh", ctypes.c_long)
                + _fields("kv", ctypes.c_void_p)
                + _fields("kvst", ctypes.c_long)
                + _fields("w freq cache pos seq bt", ctypes.c_void_p)
                + _fields("MB H R P rot", ctypes.c_int)
                + _fields("eps amp", ctypes.c_float)
                + _fields("pairs", ctypes.c_int))


class _HeadLinearArgs(ctypes.Structure):
    _fields_ = (_fields("x", ctypes.c_void_p)
                + _fields("xst xh", ctypes.c_long)
                + _fields("w out", ctypes.c_void_p)
                + _fields("ost oh", ctypes.c_long)
                + _fields("gate", ctypes.c_void_p)
                + _fields("gst gh", ctypes.c_long)
                + _fields("T H N K", ctypes.c_int))


class _LatentRowsArgs(ctypes.Structure):
    _fields_ = (_fields("q cache pos seq bt part out", ctypes.c_void_p)
                + _fields("MB rows H R P splits window", ctypes.c_int)
                + _fields("scale", ctypes.c_float)
                + _fields("sink", ctypes.c_void_p))


class _MoePlanArgs(ctypes.Structure):
    _fields_ = (_fields("z bias idx coef order tiles", ctypes.c_void_p)
                + _fields("T E top tile_rows max_tiles kind groups keep best",
                          ctypes.c_int))


class _MoeGemmArgs(ctypes.Structure):
    _fields_ = (_fields("x", ctypes.c_void_p) + _fields("xst", ctypes.c_long)
                + _fields("w out order tiles", ctypes.c_void_p)
                + _fields("top N K max_tiles", ctypes.c_int)
                + _fields("alpha limit shift", ctypes.c_float))


class _MemoryArgs(ctypes.Structure):
    _fields_ = (_fields("q k v", ctypes.c_void_p)
                + _fields("qst kst vst", ctypes.c_long)
                + _fields("gates ib fb decay log2_decay S n m seg out",
                          ctypes.c_void_p)
                + _fields("H D E", ctypes.c_int)
                + _fields("gate_cap qscale", ctypes.c_float)
                + _fields("G", ctypes.c_int)
                + _fields("skip z", ctypes.c_void_p)
                + _fields("zst", ctypes.c_long)
                + _fields("cw cb ring", ctypes.c_void_p)
                + _fields("taps C kch qch", ctypes.c_int)
                + _fields("freq", ctypes.c_void_p)
                + _fields("rot", ctypes.c_int)
                + _fields("amp kscale", ctypes.c_float))


class _ChunkArgs(ctypes.Structure):
    _fields_ = ([("a", _MemoryArgs)] + _fields("chunks first", ctypes.c_void_p)
                + _fields("n_chunks n_seg T", ctypes.c_int)
                + _fields("b i c tot cend U N P mst VT KA QA", ctypes.c_void_p)
                + _fields("norm_eps", ctypes.c_float))


# ---------------------------------------------------------------------------
# matrix products with a 32-bit result
# ---------------------------------------------------------------------------

def linear_f32(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x (T, K) @ w (N, K)^T with a float32 result (no rounding to the
    activation type): gate logits, vocabulary logits, residual projections."""
    if x.dtype == torch.float32:
        return torch.mm(x, w.t())
    return torch.mm(x, w.t(), out_dtype=torch.float32)


# ---------------------------------------------------------------------------
# residual + norm
# ---------------------------------------------------------------------------

@dataclass
class Pending:
    """A sublayer result that has not been added to the residual yet: one
    tensor, or two branches that are RMS-normed with their own weights and
    summed; ``scale`` times that.  One tensor is RMS-normed when ``w1`` is
    given, over ``groups`` equal parts each.  ``coef`` (rows, parts) makes a row the weighted sum of ``parts``
    rows of ``delta`` (rows * parts, W).  ``centred``: w1 and w2 are stored as
    their distance from one.  ``vec`` is a row added to every token.  Instead
    of ``delta``, up to two gated ``branches`` may be pending."""
    delta: Optional[torch.Tensor] = None
    delta2: Optional[torch.Tensor] = None
    w1: Optional[torch.Tensor] = None
    w2: Optional[torch.Tensor] = None
    scale: float = 1.0
    vec: Optional[torch.Tensor] = None
    coef: Optional[torch.Tensor] = None
    centred: bool = False
    groups: int = 1
    branches: Sequence["Branch"] = ()


@dataclass
class Branch:
    """A gated sublayer result: the rows of ``delta``, or with ``coef`` (rows,
    parts) their weighted sums; plus ``plus`` (rows, W); times sigmoid(gate +
    bias) of ``gate`` (rows, W) and ``bias`` (W,)."""
    delta: torch.Tensor
    coef: Optional[torch.Tensor] = None
    plus: Optional[torch.Tensor] = None
    gate: Optional[torch.Tensor] = None
    bias: Optional[torch.Tensor] = None

    @property
    def rows(self) -> int:
        return (self.delta if self.coef is None else self.coef).shape[0]

    def args(self, rows: int, W: int, dtype) -> _BranchArgs:
        parts = 1 if self.coef is None else self.coef.shape[1]
        assert self.delta.shape == (rows * parts, W)
        assert self.delta.is_contiguous() and self.delta.dtype == dtype
        a = _BranchArgs(delta=_p(self.delta), parts=parts)
        if self.coef is not None:
            assert self.coef.shape[0] == rows and self.coef.is_contiguous()
            assert self.coef.dtype == torch.float32
            a.coef = _p(self.coef)
        if self.plus is not None:
            assert self.plus.shape == (rows, W) and self.plus.dtype == dtype
            assert self.plus.is_contiguous()
            a.plus = _p(self.plus)
        if self.gate is not None:
            assert self.gate.shape == (rows, W) and self.gate.dtype == dtype
            assert self.gate.stride(1) == 1
            a.gate, a.gst = _p(self.gate), self.gate.stride(0)
        if self.bias is not None:
            assert self.bias.shape == (W,) and self.bias.dtype == dtype
            assert self.gate is not None and self.bias.is_contiguous()
            a.bias = _p(self.bias)
        return a


@dataclass
class ShortConv:
    """A causal convolution over time, one filter a channel, with the last
    inputs of every request: ``ring`` (slots, taps, C) holds the input at
    position p in place p % taps."""
    w: torch.Tensor            # (taps, C); the last row weighs the token itself
    ring: torch.Tensor
    bias: Optional[torch.Tensor] = None

    def check(self, C, dtype):
        assert self.w.shape[1] == C and self.w.is_contiguous()
        assert self.ring.shape[1:] == self.w.shape
        assert self.ring.is_contiguous() and self.w.shape[0] <= MAX_TAPS
        assert self.w.dtype == self.ring.dtype == dtype
        assert self.bias is None or (self.bias.shape == (C,)
                                     and self.bias.dtype == dtype)


def short_conv(x, conv: ShortConv, seg, chunks, silu: bool = False,
               add: bool = False,
               out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Convolve the rows of prompt portions x (T, C) and keep their last
    inputs: silu(y), or x + y, of y = bias + conv(x).  ``seg`` lists the
    portions (slot, first row, rows, context), ``chunks`` is the device form of
    ``chunk_table``."""
    T, C = x.shape
    conv.check(C, x.dtype)
    assert x.stride(1) == 1
    out = _out(out, T, C, x)
    a = _ConvArgs(x=_p(x), xst=x.stride(0), w=_p(conv.w), bias=_p(conv.bias),
                  out=_p(out), ost=C, ring=_p(conv.ring), seg=_p(seg),
                  chunks=_p(chunks), n_chunks=chunks.shape[0], chunk=CHUNK,
                  C=C, taps=conv.w.shape[0], silu=int(silu), add=int(add))
    _check(library().sv_short_conv(ctypes.byref(a),
                                   int(_aligned((C,), x, out)), _f32(x),
                                   _stream()), "short_conv")
    return out


def residual_norm(x: Optional[torch.Tensor], pending: Optional[Pending],
                  eps: float, weight: Optional[torch.Tensor] = None,
                  x0: Optional[torch.Tensor] = None, keep_x: bool = True,
                  index: Optional[torch.Tensor] = None, dtype=None,
                  centred: bool = False, copy: bool = False, groups: int = 1,
                  scale: float = 1.0, conv: Optional[ShortConv] = None,
                  batch=None):
    """Add ``pending`` to the float32 residual ``x`` (None: zero) and return
    (new x or None, RMS-normed row * weight or None, [new x; x0] or None).
    ``centred``: the weight is stored as its distance from one.  ``copy``: the
    second result is the new x itself, rounded to ``dtype``.  ``groups``: every
    one of so many equal parts is normed on its own.  ``scale`` multiplies the
    second result.  ``conv``: the second result is h + conv(h) of the rows h of
    ``batch``."""
    branches = () if pending is None else pending.branches
    src = x if pending is None else \
        branches[0].delta if branches else pending.delta
    rows, W = src.shape
    if branches:
        assert pending.delta is None and pending.coef is None and \
            pending.w1 is None and len(branches) <= 2
        rows = branches[0].rows
        assert x is None or x.shape == (rows, W)
    if pending is not None and pending.coef is not None:
        assert pending.coef.is_contiguous() and \
            pending.coef.dtype == torch.float32
        assert pending.delta2 is None and \
            pending.coef.numel() == rows
        rows = pending.coef.shape[0]
    dtype = dtype or (weight if weight is not None else x0).dtype
    f32 = _f32(src) if dtype == torch.float32 else 0
    out_rows = rows if index is None else index.shape[0]
    dev = src.device
    x_new = torch.empty(out_rows, W, dtype=torch.float32, device=dev) \
        if keep_x else None
    h = torch.empty(out_rows, W, dtype=dtype, device=dev) \
        if weight is not None or copy else None
    cat = torch.empty(out_rows, 2 * W, dtype=dtype, device=dev) \
        if x0 is not None else None
    a = _ResidualNormArgs(rows_out=out_rows, W=W, eps=eps, groups=groups,
                          p_groups=1, h_scale=scale)
    a.x, a.x_out, a.h, a.w = _p(x), _p(x_new), _p(h), _p(weight)
    a.cat, a.x0, a.index = _p(cat), _p(x0), _p(index)
    a.w_base, a.scale = float(centred), 1.0
    for i, b in enumerate(branches):
        a.br[i] = b.args(rows, W, dtype)
    a.branches = len(branches)
    if pending is not None and pending.vec is not None:
        a.vec = _p(pending.vec)
    if pending is not None and not branches:
        d = pending.delta
        assert d.is_contiguous() and d.dtype in (dtype, torch.float32)
        assert pending.delta2 is None or (
            d.dtype == dtype and pending.delta2.is_contiguous()
            and pending.delta2.shape == d.shape)
        a.delta, a.delta2 = _p(d), _p(pending.delta2)
        a.w1, a.w2 = _p(pending.w1), _p(pending.w2)
        a.coef, a.scale = _p(pending.coef), pending.scale
        a.p_groups = pending.groups
        assert pending.groups == 1 or (pending.w1 is not None
                                       and pending.delta2 is None)
        if pending.coef is not None:
            a.parts = pending.coef.shape[1]
            assert d.dtype == dtype
        a.p_base = float(pending.centred)
        a.delta_f32 = int(d.dtype == torch.float32 and
                          dtype != torch.float32)
    hc = None
    if conv is not None:
        assert weight is not None and index is None
        conv.check(W, dtype)
        hc = torch.empty_like(h)
        n = batch.portion_tokens
        assert out_rows - n == batch.singles.shape[0] and conv.bias is None
        a.conv, a.ring, a.hc = _p(conv.w), _p(conv.ring), _p(hc)
        a.singles, a.taps, a.conv_row = _p(batch.singles), conv.w.shape[0], n
    _check(library().sv_residual_norm(ctypes.byref(a), f32, _stream()),
           "residual_norm")
    if hc is not None:
        if n:
            short_conv(h[:n], conv, batch.portions, batch.chunks, add=True,
                       out=hc[:n])
        h = hc
    return x_new, h, cat


def gated_norm(o: torch.Tensor, weight: Optional[torch.Tensor],
               gate: Optional[torch.Tensor], group: int,
               eps: float, silu: bool = False,
               out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """o (T, N): every ``group`` elements divided by their root mean square,
    times weight (N,) if there is one, times sigmoid(gate (T, N)), or
    silu(gate), if there is a gate.  ``out`` may be o."""
    T, N = o.shape
    assert N % group == 0 and o.is_contiguous()
    out = _out(out, T, N, o)
    vec4 = int(group % 4 == 0)
    if gate is not None:
        assert gate.shape == o.shape and gate.stride(1) == 1
        vec4 = int(vec4 and gate.stride(0) % 4 == 0
                   and gate.storage_offset() % 4 == 0)
    _check(library().sv_gated_norm(
        ctypes.c_void_p(_p(o)), ctypes.c_void_p(_p(weight)),
        ctypes.c_void_p(_p(gate)),
        ctypes.c_long(0 if gate is None else gate.stride(0)),
        ctypes.c_void_p(_p(out)), T, N // group, group, ctypes.c_float(eps),
        int(silu), vec4, _f32(o), _stream()), "gated_norm")
    return out


def poly_norm(x: torch.Tensor, act: torch.Tensor, eps: float) -> torch.Tensor:
    """x (T, n) -> a N(x) + b N(x^2) + c N(x^3) + e of act = (a, b, c, e),
    powers element by element; N divides a row by its root mean square."""
    T, n = x.shape
    assert x.stride(1) == 1 and act.shape == (4,) and act.is_contiguous()
    assert act.dtype == x.dtype
    out = torch.empty(T, n, dtype=x.dtype, device=x.device)
    _check(library().sv_poly_norm(
        ctypes.c_void_p(_p(x)), ctypes.c_long(x.stride(0)),
        ctypes.c_void_p(_p(act)), ctypes.c_void_p(_p(out)), T, n,
        ctypes.c_float(eps), _vec4((n,), x), _f32(x), _stream()),
        "poly_norm")
    return out


def silu_mul(x: torch.Tensor) -> torch.Tensor:
    """x (T, 2 n) = [gate | up] -> silu(gate) * up (T, n)."""
    T, n = x.shape[0], x.shape[1] // 2
    assert x.stride(1) == 1 and x.shape[1] == 2 * n
    out = torch.empty(T, n, dtype=x.dtype, device=x.device)
    _check(library().sv_silu_mul(
        ctypes.c_void_p(_p(x)), ctypes.c_long(x.stride(0)),
        ctypes.c_void_p(_p(out)), T, n, _vec4((n,), x), _f32(x),
        _stream()), "silu_mul")
    return out


def relu_squared_(x: torch.Tensor) -> torch.Tensor:
    assert x.is_contiguous()
    _check(library().sv_relu_squared(ctypes.c_void_p(_p(x)),
                                     ctypes.c_long(x.numel()), _f32(x),
                                     _stream()), "relu_squared")
    return x


def gelu_tanh_(x: torch.Tensor) -> torch.Tensor:
    assert x.is_contiguous()
    _check(library().sv_gelu_tanh(ctypes.c_void_p(_p(x)),
                                  ctypes.c_long(x.numel()), _f32(x),
                                  _stream()), "gelu_tanh")
    return x


def gelu_rows_(x: torch.Tensor, table: torch.Tensor, tokens: torch.Tensor,
               at: int) -> torch.Tensor:
    """x (T, n) <- gelu(x), in its tanh form, times the columns [at, at + n)
    of table (vocab, columns) in the rows ``tokens`` (T,) int32."""
    T, n = x.shape
    assert x.is_contiguous() and table.stride(1) == 1
    assert x.dtype == table.dtype and 0 <= at <= table.shape[1] - n
    assert tokens.dtype == torch.int32 and tokens.shape == (T,)
    _check(library().sv_gelu_rows(
        ctypes.c_void_p(_p(x)), ctypes.c_void_p(_p(table)),
        ctypes.c_long(table.stride(0)), ctypes.c_void_p(_p(tokens)),
        ctypes.c_long(T), n, at, _f32(x), _stream()), "gelu_rows")
    return x


def softcap_(x: torch.Tensor, cap: float) -> torch.Tensor:
    assert x.is_contiguous() and x.dtype == torch.float32 and x.is_cuda
    _check(library().sv_softcap(ctypes.c_void_p(_p(x)),
                                ctypes.c_long(x.numel()),
                                ctypes.c_float(cap), _stream()), "softcap")
    return x


# ---------------------------------------------------------------------------
# paged attention
# ---------------------------------------------------------------------------

def _aligned(sizes, *tensors) -> bool:
    """Can rows be read in 16-byte pieces of 8 bf16 (or 2 x 4 f32)?"""
    return all(s % 8 == 0 for s in sizes) and all(
        t.stride(0) % 8 == 0 and t.storage_offset() % 8 == 0
        for t in tensors)


def _vec4(sizes, *tensors) -> int:
    return int(all(s % 4 == 0 for s in sizes) and all(
        t.stride(0) % 4 == 0 and t.storage_offset() % 4 == 0
        for t in tensors))


def _check_cache(q, k, v, kc, vc, H):
    G, D, E = kc.shape[1], kc.shape[3], vc.shape[3]
    assert kc.shape[:3] == vc.shape[:3] and kc.shape[2] == PAGE_SIZE
    assert kc.is_contiguous() and vc.is_contiguous() and H % G == 0
    assert q.shape[1] == H * D and k.shape[1] == G * D and \
        v.shape[1] == G * E
    assert q.stride(1) == k.stride(1) == v.stride(1) == 1
    assert q.dtype == k.dtype == v.dtype == kc.dtype == vc.dtype
    if max(D, E) > MAX_HEAD_DIM:
        raise ValueError(f"head size {max(D, E)} > {MAX_HEAD_DIM}")
    return G, D, E


def _out(out, rows, cols, like):
    if out is None:
        return torch.empty(rows, cols, dtype=like.dtype, device=like.device)
    assert out.shape == (rows, cols) and out.is_contiguous() and \
        out.dtype == like.dtype
    return out


def kv_append(k, v, kc, vc, pos, seq, block_table):
    """Write k (T, G*D) and v (T, G*E) at positions ``pos`` of the requests
    ``seq`` (int32, row of the block table)."""
    G, D, E = kc.shape[1], kc.shape[3], vc.shape[3]
    T = k.shape[0]
    assert pos.shape[0] == T and seq.shape[0] == T
    _check(library().sv_kv_append(
        ctypes.c_void_p(_p(k)), ctypes.c_void_p(_p(v)),
        ctypes.c_long(k.stride(0)), ctypes.c_long(v.stride(0)),
        ctypes.c_void_p(_p(kc)), ctypes.c_void_p(_p(vc)),
        ctypes.c_void_p(_p(pos)), ctypes.c_void_p(_p(seq)),
        ctypes.c_void_p(_p(block_table)), block_table.shape[1], T, G, D, E,
        int(_aligned((D, E), k, v)), _f32(k), _stream()), "kv_append")


@dataclass
class QkvPrep:
    """What happens to queries, keys and values before they are attended and
    cached: the first elements of a head turn in neighbouring pairs, queries
    and keys are RMS-normed a head, queries grow with their position, values
    take a share of another layer's."""
    freq: Optional[torch.Tensor] = None    # (dims / 2,) float64 rad a position
    norm: bool = False
    q_norm: Optional[torch.Tensor] = None  # (D,) weights of the norm
    k_norm: Optional[torch.Tensor] = None
    eps: float = 0.0
    temp_coef: float = 0.0                 # q *= 1 + coef ln(floor((p + 1) /
    temp_every: int = 0                    #   every) + 1), if every > 0
    first: Optional[torch.Tensor] = None   # (T, G * E)
    mix: Optional[torch.Tensor] = None     # one number: v + mix (first - v)


@dataclass
class ScoreMod:
    """Of the scores s = q.k scale and their softmax: s *= temp[h];
    s = cap tanh(s / cap); s -= slope[h] distance; exp(sink[h]) joins the
    denominator; the output is multiplied by sigmoid(gate[row, h])."""
    temp: Optional[torch.Tensor] = None    # (H,)
    cap: float = 0.0
    slope: Optional[torch.Tensor] = None   # (H,) float32
    sink: Optional[torch.Tensor] = None    # (H,)
    gate: Optional[torch.Tensor] = None    # (T, H)

    def rows(self, a, b):
        """The same for rows [a, b) of the batch."""
        return self if self.gate is None else replace(self,
                                                      gate=self.gate[a:b])


def _score_args(mod: Optional[ScoreMod], q, H) -> _ScoreArgs:
    if mod is None:
        return _ScoreArgs()
    for t in (mod.temp, mod.sink):
        assert t is None or (t.shape == (H,) and t.dtype == q.dtype
                             and t.is_cuda and t.is_contiguous())
    assert mod.slope is None or (mod.slope.shape == (H,) and mod.slope.is_cuda
                                 and mod.slope.dtype == torch.float32)
    a = _ScoreArgs(temp=_p(mod.temp), sink=_p(mod.sink), slope=_p(mod.slope),
                   cap=mod.cap)
    if mod.gate is not None:
        assert mod.gate.shape == (q.shape[0], H) and mod.gate.stride(1) == 1
        assert mod.gate.dtype == q.dtype
        a.gate, a.gst = _p(mod.gate), mod.gate.stride(0)
    return a


def qkv_append(q, k, v, kc, vc, pos, seq, block_table, heads: int,
               prep: QkvPrep):
    """Prepare q (T, H*D) in place and write the prepared k and v at positions
    ``pos`` of the requests ``seq``."""
    G, D, E = _check_cache(q, k, v, kc, vc, heads)
    T = q.shape[0]
    assert pos.shape[0] == seq.shape[0] == T
    a = _QkvArgs(q=_p(q), k=_p(k), v=_p(v), qst=q.stride(0), kst=k.stride(0),
                 vst=v.stride(0), kc=_p(kc), vc=_p(vc), pos=_p(pos),
                 seq=_p(seq), bt=_p(block_table), MB=block_table.shape[1],
                 T=T, H=heads, G=G, D=D, E=E, norm=int(prep.norm),
                 temp_every=prep.temp_every, temp_coef=prep.temp_coef,
                 eps=prep.eps)
    tensors = [q, k, v]
    if prep.freq is not None:
        assert prep.freq.dtype == torch.float64 and prep.freq.is_cuda
        a.freq, a.rot = _p(prep.freq), 2 * prep.freq.shape[0]
    for name, w in (("qw", prep.q_norm), ("kw", prep.k_norm)):
        if w is not None:
            assert w.shape == (D,) and w.dtype == q.dtype and prep.norm
            setattr(a, name, _p(w))
    if prep.first is not None:
        f = prep.first
        assert f.shape == v.shape and f.stride(1) == 1 and f.dtype == v.dtype
        assert prep.mix.numel() == 1 and prep.mix.dtype == v.dtype
        a.first, a.fst, a.mix = _p(f), f.stride(0), _p(prep.mix)
        tensors.append(f)
    _check(library().sv_qkv_append(
        ctypes.byref(a), int(_aligned((D, E), *tensors)), _f32(q), _stream()),
        "qkv_append")


def _row_splits(target: int, units: int, max_keys: int, per: int) -> int:
    """Workgroups that share a row: enough for ``target`` of them, each with
    about ``per`` keys or more."""
    return max(1, min(target // max(1, units), -(-max_keys // per), 64))


def attn_rows(q, k, v, kc, vc, pos, seq, block_table, heads: int,
              scale: float, window: int = 0, keep: int = 0,
              append: bool = True, max_keys: int = 0,
              out: Optional[torch.Tensor] = None,
              mod: Optional[ScoreMod] = None) -> torch.Tensor:
    """One query row per request row: decoding.  ``append`` also writes the
    row's own k/v into the cache (without it they must be there already).
    ``max_keys`` bounds the visible keys of any row (it only sets how many
    workgroups share a row)."""
    G, D, E = _check_cache(q, k, v, kc, vc, heads)
    rows = q.shape[0]
    assert pos.shape[0] == rows and seq.shape[0] == rows
    if window > 0:
        max_keys = min(max_keys, window + keep) if max_keys else window + keep
    splits = _row_splits(1024, rows * G, max_keys, 128)
    out = _out(out, rows, heads * E, q)
    part = torch.empty(rows * heads * splits * (E + 2), dtype=torch.float32,
                       device=q.device) if splits > 1 else None
    a = _RowsArgs(q=_p(q), k=_p(k), v=_p(v), qst=q.stride(0),
                  kst=k.stride(0), vst=v.stride(0), kc=_p(kc), vc=_p(vc),
                  kcs=D, vcs=E,
                  pos=_p(pos), seq=_p(seq), bt=_p(block_table),
                  part=_p(part), out=_p(out), MB=block_table.shape[1],
                  rows=rows, H=heads, G=G, D=D, E=E, splits=splits,
                  append=int(append), window=window, keep=keep, scale=scale,
                  mod=_score_args(mod, q, heads))
    _check(library().sv_attn_rows(ctypes.byref(a),
                                  int(_aligned((D, E), q, k, v)), _f32(q),
                                  _stream()), "attn_rows")
    return out


def attn_tiles_supported(q, kc, vc) -> bool:
    D, E = kc.shape[3], vc.shape[3]
    return (q.dtype == torch.bfloat16 and max(D, E) <= 256
            and _aligned((D, E), q))


def attn_portions(q, k, v, kc, vc, pos, seq, block_table, tiles, heads: int,
                  scale: float, window: int = 0, keep: int = 0,
                  append: bool = True, max_keys: int = 0,
                  out: Optional[torch.Tensor] = None,
                  mod: Optional[ScoreMod] = None) -> torch.Tensor:
    """Prompt portions: append k/v (unless they are there), then causal
    attention of every row over its request's cache.  ``tiles`` (n, 4) int32
    lists (request, first row, rows <= 128, position of the first row)."""
    G, D, E = _check_cache(q, k, v, kc, vc, heads)
    if append:
        kv_append(k, v, kc, vc, pos, seq, block_table)
    if not attn_tiles_supported(q, kc, vc):
        return attn_rows(q, k, v, kc, vc, pos, seq, block_table, heads,
                         scale, window, keep, append=False,
                         max_keys=max_keys, out=out, mod=mod)
    out = _out(out, q.shape[0], heads * E, q)
    a = _TilesArgs(q=_p(q), qst=q.stride(0), kc=_p(kc), vc=_p(vc),
                   kpage=G * PAGE_SIZE * D, khead=PAGE_SIZE * D, krow=D,
                   vpage=G * PAGE_SIZE * E, vhead=PAGE_SIZE * E, vrow=E,
                   tiles=_p(tiles), bt=_p(block_table), out=_p(out),
                   MB=block_table.shape[1], H=heads, G=G, D=D, E=E, DS=D,
                   window=window, keep=keep, scale=scale,
                   mod=_score_args(mod, q, heads))
    _check(library().sv_attn_tiles(ctypes.byref(a), tiles.shape[0],
                                   _stream()), "attn_tiles")
    return out


def ragged_attention(q, k, v, batch, pool, heads: int, scale: float,
                     window: int = 0, keep: int = 0,
                     prep: Optional[QkvPrep] = None,
                     mod: Optional[ScoreMod] = None) -> torch.Tensor:
    """Attention of a packed batch over its cache pool: portions first, then
    single tokens, into one (T, heads * E) tensor.  ``prep`` changes q in
    place."""
    kc, vc = pool
    T, n = q.shape[0], batch.portion_tokens
    out = torch.empty(T, heads * vc.shape[3], dtype=q.dtype, device=q.device)
    args = dict(heads=heads, scale=scale, window=window, keep=keep,
                max_keys=batch.max_keys, append=prep is None)
    if prep is not None:
        qkv_append(q, k, v, kc, vc, batch.pos, batch.seq, batch.block_table,
                   heads, prep)
    if n:
        attn_portions(q[:n], k[:n], v[:n], kc, vc, batch.pos[:n],
                      batch.seq[:n], batch.block_table, batch.tiles,
                      out=out[:n], mod=mod and mod.rows(0, n), **args)
    if n < T:
        attn_rows(q[n:], k[n:], v[n:], kc, vc, batch.pos[n:], batch.seq[n:],
                  batch.block_table, out=out[n:], mod=mod and mod.rows(n, T),
                  **args)
    return out


def rope_rows_(q, k, cos, sin, pos, dim: int, max_pos: int):
    """Rotate the heads of q and k (rotate-half) in place, each row at its
    own position; cos/sin (positions, dim / 2) float32."""
    if max_pos > cos.shape[0]:
        raise ValueError(f"position {max_pos - 1} is outside the rotary "
                         f"table of {cos.shape[0]}")
    assert cos.dtype == sin.dtype == torch.float32 and cos.is_contiguous()
    assert sin.is_contiguous() and cos.shape[1] * 2 == dim
    assert q.stride(1) == k.stride(1) == 1 and pos.shape[0] == q.shape[0]
    vp, lg = ctypes.c_void_p, ctypes.c_long
    _check(library().sv_rope_rows(
        vp(_p(q)), lg(q.stride(0)), q.shape[1] // dim, vp(_p(k)),
        lg(k.stride(0)), k.shape[1] // dim, vp(_p(cos)), vp(_p(sin)),
        vp(_p(pos)), q.shape[0], dim, _f32(q), _stream()), "rope_rows")


# ---------------------------------------------------------------------------
# recurrent matrix memories
# ---------------------------------------------------------------------------

@dataclass
class DecayGate:
    """S <- decay S + k v^T; q, k and v pass through silu."""
    decay: torch.Tensor        # (H,) float32
    log2_decay: torch.Tensor   # (H,) float32


@dataclass
class ExpGate:
    """Exponential input and forget gates with a running maximum."""
    raw: torch.Tensor          # (T, 2H) float32: i then f projections
    i_bias: torch.Tensor       # (H,)
    f_bias: torch.Tensor       # (H,)
    cap: float
    qscale: float


@dataclass
class TimeGate:
    """A time step from a projection: dt = softplus(raw + bias), S <-
    exp(-exp(A_log) dt) S + dt k v^T; o = (S^T q + skip v) silu(z).  Heads share
    q and k in groups.  ``conv``: q, k and v of single tokens have not passed
    their convolution and silu yet; its channels are v's, then k's, then q's."""
    raw: torch.Tensor          # (T, H) float32
    bias: torch.Tensor         # (H,)
    A_log: torch.Tensor        # (H,)
    skip: torch.Tensor         # (H,)
    z: torch.Tensor            # (T, H * E)
    conv: Optional[ShortConv] = None


@dataclass
class TurnGate:
    """S <- decay S + kscale k v^T, with q and k rotated at their position:
    elements i and i + dims / 2 of a head turn together."""
    decay: torch.Tensor        # (H,) float32
    log2_decay: torch.Tensor   # (H,) float32
    kscale: float
    freq: torch.Tensor         # (dims / 2,) float64 rad a position
    amplitude: float = 1.0     # of cos and sin

    @staticmethod
    def norm_fits(dtype, D: int, E: int, *tensors) -> bool:
        """Can the chunk kernels norm and gate the heads as well?"""
        return (dtype == torch.bfloat16 and D <= 256
                and E <= (128 if D <= 128 else 64)
                and _aligned((D, E), *tensors))


_GATINGS = {DecayGate: 0, ExpGate: 1, TimeGate: 2, TurnGate: 3}


def chunk_table(segments):
    """Chunks of prompt portions: rows (segment, first row, rows, does a
    state come in) and the first chunk of every segment, from rows (slot,
    first row, rows, context)."""
    rows, first = [], [0]
    for i, (_, r0, n, ctx) in enumerate(segments):
        for at in range(0, n, CHUNK):
            rows.append((i, r0 + at, min(CHUNK, n - at),
                         int(at > 0 or ctx > 0)))
        first.append(len(rows))
    return rows, first


def memory_mix(q, k, v, gate, S, n, m, seg, heads: int,
               chunks: Optional[torch.Tensor] = None,
               chunk_first: Optional[torch.Tensor] = None,
               out: Optional[torch.Tensor] = None,
               silu_gate: Optional[torch.Tensor] = None,
               eps: float = 0.0) -> torch.Tensor:
    """Run a matrix memory over segments of a ragged batch.  q, k (T, H*D),
    v (T, H*E) — q, k (T, G*D) for a TimeGate; S (slots, H, D, E) float32; n (slots, H, ceil(E/32), D) and
    m (slots, H, ceil(E/32)) float32 for an ExpGate.  ``seg`` (n, 4) int32
    lists (slot, first row, rows, context); rows count from the start of
    the tensors, so portions and single tokens of one batch can be run by
    two calls into one ``out``.  With the device form of
    ``chunk_table`` the 256-token MFMA kernels run where they apply; with a
    TurnGate that ``norm_fits`` they also divide every head of the output by
    its root mean square and multiply it by silu(``silu_gate`` (T, H*E))."""
    D, E = S.shape[2], S.shape[3]
    T = q.shape[0]
    assert q.shape[1] == k.shape[1] and v.shape[1] == heads * E
    assert q.stride(1) == k.stride(1) == v.stride(1) == 1
    assert S.is_contiguous() and S.dtype == torch.float32
    assert S.shape[1] == heads
    if D > MAX_HEAD_DIM:
        raise ValueError(f"key size {D} > {MAX_HEAD_DIM}")
    out = _out(out, T, heads * E, q)
    a = _MemoryArgs(q=_p(q), k=_p(k), v=_p(v), qst=q.stride(0),
                    kst=k.stride(0), vst=v.stride(0), S=_p(S), seg=_p(seg),
                    out=_p(out), H=heads, D=D, E=E, gate_cap=1.0, qscale=1.0,
                    G=q.shape[1] // D)
    assert q.shape[1] == a.G * D and heads % a.G == 0
    gating = _GATINGS[type(gate)]
    gated, timed = isinstance(gate, ExpGate), isinstance(gate, TimeGate)
    turned = isinstance(gate, TurnGate)
    assert timed or a.G == heads
    strided = [q, k, v]
    if timed:
        for t in (gate.bias, gate.A_log, gate.skip):
            assert t.shape == (heads,) and t.dtype == q.dtype
        assert gate.raw.shape == (T, heads) and gate.raw.is_contiguous() \
            and gate.raw.dtype == torch.float32
        assert gate.z.shape == v.shape and gate.z.stride(1) == 1 \
            and gate.z.dtype == v.dtype
        a.gates, a.ib, a.fb = _p(gate.raw), _p(gate.bias), _p(gate.A_log)
        a.skip, a.z, a.zst = _p(gate.skip), _p(gate.z), gate.z.stride(0)
        strided.append(gate.z)
        if gate.conv is not None:
            assert chunks is None      # one token a segment
            a.kch, a.qch = heads * E, heads * E + k.shape[1]
            a.C, a.taps = a.qch + q.shape[1], gate.conv.w.shape[0]
            gate.conv.check(a.C, q.dtype)
            a.cw, a.cb = _p(gate.conv.w), _p(gate.conv.bias)
            a.ring = _p(gate.conv.ring)
    elif gated:
        nt = (E + 31) // 32
        assert n.shape[1:] == (heads, nt, D) and m.shape[1:] == (heads, nt)
        assert gate.raw.shape == (T, 2 * heads) and \
            gate.raw.is_contiguous() and gate.raw.dtype == torch.float32
        assert gate.i_bias.dtype == gate.f_bias.dtype == q.dtype
        a.gates, a.ib, a.fb = _p(gate.raw), _p(gate.i_bias), _p(gate.f_bias)
        a.n, a.m = _p(n), _p(m)
        a.gate_cap, a.qscale = gate.cap, gate.qscale
    else:
        assert gate.decay.shape == (heads,)
        a.decay, a.log2_decay = _p(gate.decay), _p(gate.log2_decay)
    if turned:
        assert gate.freq.dtype == torch.float64 and gate.freq.is_cuda
        a.freq, a.rot = _p(gate.freq), 2 * gate.freq.shape[0]
        a.amp, a.kscale = gate.amplitude, gate.kscale
        if a.rot > D:
            raise ValueError(f"{a.rot} of {D} elements turn")
    if silu_gate is not None:
        assert turned and chunks is not None
        assert gate.norm_fits(q.dtype, D, E, q, k, v, silu_gate)
        assert silu_gate.shape == v.shape and silu_gate.stride(1) == 1 \
            and silu_gate.dtype == v.dtype
        a.z, a.zst = _p(silu_gate), silu_gate.stride(0)
    lib = library()
    if (chunks is not None and q.dtype == torch.bfloat16 and D <= 256
            and _aligned((D, E), *strided)):
        nc = chunks.shape[0]
        assert chunk_first.shape[0] == seg.shape[0] + 1
        f32 = dict(dtype=torch.float32, device=q.device)
        U = torch.empty(nc, heads, E, D, **f32)
        P = torch.empty(nc, heads, 3, E, D, dtype=torch.bfloat16,
                        device=q.device)
        VT = torch.empty(nc, heads, E, CHUNK, dtype=torch.bfloat16,
                         device=q.device)
        KA = torch.empty(T, heads * D, dtype=q.dtype, device=q.device) \
            if isinstance(gate, DecayGate) else None
        if turned:
            KA, QA = torch.empty(2, 2, T, heads * D, dtype=q.dtype,
                                 device=q.device)
        x = _ChunkArgs(a=a, chunks=_p(chunks), first=_p(chunk_first),
                       n_chunks=nc, n_seg=seg.shape[0], T=T, U=_p(U),
                       P=_p(P), VT=_p(VT), KA=_p(KA), norm_eps=eps)
        if turned:
            x.QA = _p(QA)
        if timed:
            bic = torch.empty(2, heads, T, **f32)
            small = torch.empty(nc, heads, 4, **f32)
            x.b, x.i, x.tot = _p(bic[0]), _p(bic[1]), _p(small)
        elif gated:
            bic = torch.empty(3, heads, T, **f32)
            small = torch.empty(nc, heads, 6 + D, **f32)
            x.b, x.i, x.c = (_p(t) for t in bic)
            flat, nh = small.view(-1), nc * heads
            x.tot, x.cend = _p(flat), _p(flat[4 * nh:])
            x.mst, x.N = _p(flat[5 * nh:]), _p(flat[6 * nh:])
        st = lib.sv_memory_chunks(ctypes.byref(x), gating, _stream())
    else:
        st = lib.sv_memory_steps(ctypes.byref(a), seg.shape[0], gating,
                                 _f32(q), _stream())
    _check(st, "memory_mix")
    return out


def decay_gate(decay, device) -> DecayGate:
    d = torch.tensor([float(x) for x in decay], dtype=torch.float64)
    # finite for a decay of zero: 0 tokens apart must still weigh 2^0
    log2 = torch.log2(d).clamp(min=-1e4)
    return DecayGate(d.float().to(device), log2.float().to(device))


# ---------------------------------------------------------------------------
# latent attention
# ---------------------------------------------------------------------------

@dataclass
class KeySpans:
    """The keys that the prompt portions of a step see, gathered page after
    page into a workspace."""
    pages: torch.Tensor        # (n,) cache page of every workspace page
    table: torch.Tensor        # (portions, width) position / 64 -> its page


def key_spans(portions, block_table, window: int):
    """Host form of KeySpans: (pages, table) as lists of int from portions
    (slot, first row, rows, context) and their block-table rows."""
    pages, table = [], []
    for (_, _, n, ctx), row in zip(portions, block_table):
        a = max(0, ctx - window + 1) // PAGE_SIZE if window > 0 else 0
        b = (ctx + n - 1) // PAGE_SIZE
        places = [0] * len(row)
        for p in range(a, b + 1):
            places[p] = len(pages)
            pages.append(int(row[p]))
        table.append(places)
    return pages, table


def rotary_frequencies(base: float, dims: int, device,
                       scaling: Optional[dict] = None) -> torch.Tensor:
    """Radians a position of every rotated pair, float64.  ``scaling`` (factor,
    low, high, original): a pair that turns less than ``low`` times in
    ``original`` positions is slowed by ``factor``, one that turns more than
    ``high`` times is kept, those between are interpolated."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    f = torch.pow(torch.tensor(base, dtype=torch.float64), -2.0 * i / dims)
    if scaling:
        low, high = scaling["low"], scaling["high"]
        turns = scaling["original"] * f / (2.0 * math.pi)
        keep = ((turns - low) / (high - low)).clamp(0.0, 1.0) \
            if high > low else (turns > low).double()
        f = f * (keep + (1.0 - keep) / scaling["factor"])
    return f.to(device)


def yarn_frequencies(base: float, dims: int, device, scaling: dict):
    """Radians a position of every rotated pair, float64, and the amplitude
    of cos and sin.  ``scaling`` (factor, original, fast, slow): pairs that turn
    more than ``fast`` times in ``original`` positions are kept, those that turn
    less than ``slow`` times are slowed by ``factor``; between them, pair by
    pair, linearly from one to the other."""
    f = rotary_frequencies(base, dims, "cpu")

    def pair(turns):
        return dims * math.log(scaling["original"] / (2 * math.pi * turns)) \
            / (2 * math.log(base))

    lo = max(math.floor(pair(scaling["fast"])), 0)
    hi = min(math.ceil(pair(scaling["slow"])), dims - 1)
    i = torch.arange(dims // 2, dtype=torch.float64)
    slow = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
    f = f / scaling["factor"] * slow + f * (1.0 - slow)
    return f.to(device), 0.1 * math.log(scaling["factor"]) + 1.0


@dataclass
class LatentWeights:
    norm: torch.Tensor         # (rank,) of the latents
    absorb: torch.Tensor       # (H, rank, dim): query -> latent space
    expand: torch.Tensor       # (H * dim + H * vdim, rank): keys, values
    freq: torch.Tensor         # (rot / 2,) float64 rad a position
    amplitude: float = 1.0     # of cos and sin
    pairs: bool = False        # neighbours turn together, not halves
    sink: Optional[torch.Tensor] = None   # (H,) joins the denominator


def latent_append(q, rot_at: int, q_step: int, qr, qr_at: int, qr_step: int,
                  kv, w: LatentWeights, cache, pos, seq, block_table,
                  heads: int, eps: float):
    """Norm the latents of kv (T, rank + P), rotate the shared key, write
    both into the cache (pages, 64, rank + P); rotate columns [rot_at, + P) of
    every head of q (heads ``q_step`` apart) into those at ``qr_at`` of qr."""
    T, R = q.shape[0], w.norm.shape[0]
    P = cache.shape[2] - R
    half = w.freq.shape[0]
    assert kv.shape == (T, R + P) and cache.shape[1] == PAGE_SIZE
    assert cache.is_contiguous() and 2 * half <= P
    assert w.freq.dtype == torch.float64 and w.freq.is_cuda
    assert q.stride(1) == qr.stride(1) == kv.stride(1) == 1
    assert q.dtype == qr.dtype == kv.dtype == cache.dtype == w.norm.dtype
    assert (heads - 1) * q_step + rot_at + P <= q.shape[1]
    assert (heads - 1) * qr_step + qr_at + P <= qr.shape[1]
    assert pos.shape[0] == seq.shape[0] == T == qr.shape[0]
    size = q.element_size()
    a = _LatentAppendArgs(
        q=_p(q) + rot_at * size, qst=q.stride(0), qh=q_step,
        qr=_p(qr) + qr_at * size, qrst=qr.stride(0), qrh=qr_step, kv=_p(kv),
        kvst=kv.stride(0), w=_p(w.norm), freq=_p(w.freq), cache=_p(cache),
        pos=_p(pos), seq=_p(seq), bt=_p(block_table),
        MB=block_table.shape[1], H=heads, R=R, P=P, rot=2 * half, eps=eps,
        amp=w.amplitude, pairs=int(w.pairs))
    _check(library().sv_latent_append(ctypes.byref(a), T, _f32(q),
                                      _stream()), "latent_append")


def head_linear(x, x_step: int, w, out, out_step: int,
                gate: Optional[torch.Tensor] = None):
    """out[t, h * out_step + n] = sum_k x[t, h * x_step + k] w[h, n, k], times
    sigmoid(gate[t, h * N + n])."""
    H, N, K = w.shape
    T = x.shape[0]
    assert w.is_contiguous() and x.stride(1) == out.stride(1) == 1
    assert x.dtype == w.dtype == out.dtype and out.shape[0] == T
    assert (H - 1) * x_step + K <= x.shape[1]
    assert (H - 1) * out_step + N <= out.shape[1]
    a = _HeadLinearArgs(x=_p(x), xst=x.stride(0), xh=x_step, w=_p(w),
                        out=_p(out), ost=out.stride(0), oh=out_step,
                        T=T, H=H, N=N, K=K)
    mfma = x.dtype == torch.bfloat16 and K >= 8 and N >= 4 and N % 4 == 0 \
        and _aligned((K, x_step, out_step), x, out)
    if gate is not None:
        assert gate.shape == (T, H * N) and gate.stride(1) == 1
        assert gate.dtype == x.dtype
        a.gate, a.gst, a.gh = _p(gate), gate.stride(0), N
        mfma = mfma and _aligned((), gate)
    _check(library().sv_head_linear(ctypes.byref(a), int(mfma), _f32(x),
                                    _stream()), "head_linear")
    return out


def latent_rows_supported(dtype, rank: int, shared: int) -> bool:
    return (dtype == torch.bfloat16 and rank % 8 == 0 and shared % 8 == 0
            and rank <= 512 and shared <= 64)


def latent_rows(q, cache, rank: int, pos, seq, block_table, heads: int,
                scale: float, window: int = 0, max_keys: int = 0,
                sink: Optional[torch.Tensor] = None):
    """Absorbed queries q (rows, H * (rank + P)) over the cached rows, which
    hold the rows' own keys already -> (rows, H * rank) sums of latents.
    exp(sink[h]) joins the denominator."""
    rows, D = q.shape[0], cache.shape[2]
    assert q.is_contiguous() and q.shape[1] == heads * D
    assert cache.is_contiguous() and cache.shape[1] == PAGE_SIZE
    assert q.dtype == cache.dtype and pos.shape[0] == seq.shape[0] == rows
    if D > MAX_LATENT_ROW:
        raise ValueError(f"latent row of {D} > {MAX_LATENT_ROW}")
    mod = _score_args(ScoreMod(sink=sink), q, heads)
    if window > 0:
        max_keys = min(max_keys, window) if max_keys else window
    out = torch.empty(rows, heads * rank, dtype=q.dtype, device=q.device)
    fast = latent_rows_supported(q.dtype, rank, D - rank)
    splits = _row_splits(512, rows * -(-heads // 32), max_keys, 128) if fast \
        else _row_splits(1024, rows, max_keys, 128)
    part = torch.empty(rows * heads * splits * (rank + 2),
                       dtype=torch.float32, device=q.device) \
        if splits > 1 else None
    if fast:
        a = _LatentRowsArgs(
            q=_p(q), cache=_p(cache), pos=_p(pos), seq=_p(seq),
            bt=_p(block_table), part=_p(part), out=_p(out),
            MB=block_table.shape[1], rows=rows, H=heads, R=rank, P=D - rank,
            splits=splits, window=window, scale=scale, sink=mod.sink)
        _check(library().sv_latent_rows(ctypes.byref(a), _stream()),
               "latent_rows")
        return out
    # one key/value head whose value is the front of its key
    a = _RowsArgs(q=_p(q), k=_p(q), v=_p(q), qst=q.stride(0),
                  kst=q.stride(0), vst=q.stride(0), kc=_p(cache),
                  vc=_p(cache), kcs=D, vcs=D, pos=_p(pos), seq=_p(seq),
                  bt=_p(block_table), part=_p(part), out=_p(out),
                  MB=block_table.shape[1], rows=rows, H=heads, G=1, D=D,
                  E=rank, splits=splits, append=0, window=window, keep=0,
                  scale=scale, mod=mod)
    _check(library().sv_attn_rows(ctypes.byref(a),
                                  int(_aligned((D, rank), q)), _f32(q),
                                  _stream()), "attn_rows")
    return out


def latent_tiles_supported(q, gate, dim, vdim, rank, shared) -> bool:
    return (q.dtype == torch.bfloat16 and dim + shared <= 256
            and vdim <= 256
            and _aligned((dim, vdim, rank, shared), q)
            and (gate is None or _aligned((), gate)))


def latent_portions(q, gate, cache, w: LatentWeights, batch,
                    spans: KeySpans, heads: int, dim: int, vdim: int,
                    scale: float, window: int, out):
    """Prompt portions with rotated queries q (T, H * (dim + P)): gather the
    visible rows, make all heads' keys and values with one product, attend."""
    R = w.norm.shape[0]
    P = cache.shape[2] - R
    n = spans.pages.shape[0]
    ws = torch.empty(n * PAGE_SIZE, R + P, dtype=q.dtype, device=q.device)
    _check(library().sv_latent_gather(
        ctypes.c_void_p(_p(cache)), ctypes.c_void_p(_p(ws)),
        ctypes.c_void_p(_p(spans.pages)), n,
        PAGE_SIZE * (R + P) * q.element_size(), _stream()), "latent_gather")
    kv = torch.mm(ws[:, :R], w.expand.t())
    return expanded_attention(q, gate, kv, ws, batch.tiles, spans, heads,
                              dim, vdim, scale, window, out, w.sink)


def expanded_attention(q, gate, kv, ws, tiles, spans: KeySpans, heads: int,
                       dim: int, vdim: int, scale: float, window: int, out,
                       sink: Optional[torch.Tensor] = None):
    """Query tiles over keys and values kv (rows, H * dim + H * vdim) of the
    workspace rows ws (rows, rank + P), whose last columns end every key."""
    P = q.shape[1] // heads - dim
    R = ws.shape[1] - P
    assert q.shape[1] == heads * (dim + P) and q.stride(1) == 1
    assert kv.shape == (spans.pages.shape[0] * PAGE_SIZE,
                        heads * (dim + vdim)) and kv.is_contiguous()
    assert ws.shape[0] == kv.shape[0] and ws.is_contiguous()
    assert out.shape == (q.shape[0], heads * vdim) and out.is_contiguous()
    row, size = kv.shape[1], q.element_size()
    a = _TilesArgs(q=_p(q), qst=q.stride(0), kc=_p(kv),
                   vc=_p(kv) + heads * dim * size, kr=_p(ws) + R * size,
                   kpage=PAGE_SIZE * row, khead=dim, krow=row,
                   vpage=PAGE_SIZE * row, vhead=vdim, vrow=row, rrow=R + P,
                   tiles=_p(tiles), bt=_p(spans.table), out=_p(out),
                   MB=spans.table.shape[1], H=heads, G=heads, D=dim + P,
                   E=vdim, DS=dim, window=window, keep=0, scale=scale,
                   mod=_score_args(ScoreMod(sink=sink), q, heads))
    if gate is not None:
        assert gate.shape == out.shape and gate.stride(1) == 1
        a.gate, a.gst = _p(gate), gate.stride(0)
    _check(library().sv_attn_tiles(ctypes.byref(a), tiles.shape[0],
                                   _stream()), "attn_tiles")
    return out


def latent_attention(q, kv, gate, batch, cache, w: LatentWeights, heads: int,
                     dim: int, vdim: int, scale: float, eps: float,
                     window: int = 0) -> torch.Tensor:
    """Latent attention of a packed batch.  q (T, H * (dim + P)) head by head
    [unrotated | rotated], kv (T, rank + P), gate (T, H * vdim) or None ->
    (T, H * vdim), times sigmoid(gate)."""
    T, R = q.shape[0], w.norm.shape[0]
    D = cache.shape[2]
    P = D - R
    out = torch.empty(T, heads * vdim, dtype=q.dtype, device=q.device)
    n = batch.portion_tokens
    spans = batch.spans.get(window)
    if spans is None or not latent_tiles_supported(q, gate, dim, vdim, R, P):
        n = 0
    if n:
        g = None if gate is None else gate[:n]
        latent_append(q[:n], dim, dim + P, q[:n], dim, dim + P, kv[:n], w,
                      cache, batch.pos[:n], batch.seq[:n], batch.block_table,
                      heads, eps)
        latent_portions(q[:n], g, cache, w, batch, spans, heads, dim, vdim,
                        scale, window, out[:n])
    if n < T:
        at = (batch.pos[n:], batch.seq[n:], batch.block_table)
        ql = torch.empty(T - n, heads * D, dtype=q.dtype, device=q.device)
        latent_append(q[n:], dim, dim + P, ql, R, D, kv[n:], w, cache, *at,
                      heads, eps)
        head_linear(q[n:], dim + P, w.absorb, ql, D)
        lat = latent_rows(ql, cache, R, *at, heads, scale, window,
                          batch.max_keys, w.sink)
        head_linear(lat, R, w.expand[heads * dim:].view(heads, vdim, R),
                    out[n:], vdim, None if gate is None else gate[n:])
    return out


# ---------------------------------------------------------------------------
# mixture of experts
# ---------------------------------------------------------------------------

# kernels of the grouped products, and the most slots of their tiles
MOE_PLAIN, MOE_STREAM = 0, 1
MOE_TILES = (2, 3, 4, 5)
MOE_TILE_ROWS = (32, 32, 32, 64, 128, 256)


def moe_kernel(pairs: int, experts: int) -> int:
    """The fastest kernel for ``pairs`` spread over ``experts`` (measured)."""
    rows = pairs / experts
    if rows < 4:
        return MOE_STREAM
    return MOE_TILES[sum(rows >= r for r in (24, 112, 160))]


@dataclass
class Routing:
    """How logits choose experts.  Plain: the largest z + bias, weights a
    softmax over the chosen.  ``sigmoid``: the largest sigmoid(z) + bias,
    weights the chosen sigmoids over their sum.  ``softmax``: the largest z +
    bias, weights a softmax over all experts, not scaled to a sum of one.  With
    several ``groups`` of neighbours only the experts of the ``keep`` best can
    be chosen; a group counts the sum of its ``best`` (one or two) largest."""
    top: int
    sigmoid: bool = False
    groups: int = 1
    keep: int = 1
    softmax: bool = False
    best: int = 2

    @property
    def kind(self) -> int:
        return 2 if self.softmax else int(self.sigmoid)

    def check(self, experts: int):
        g = self.groups
        if experts > MAX_EXPERTS or not 1 <= self.top <= min(64, experts):
            raise ValueError(f"{self.top} of {experts} experts")
        if not 1 <= g <= 64 or experts % g or not 1 <= self.keep <= g or \
                self.keep * (experts // g) < self.top:
            raise ValueError(f"{self.top} experts from {self.keep} of {g} "
                             f"groups of {experts}")
        if self.best not in (1, 2) or (self.sigmoid and self.softmax):
            raise ValueError(f"routing {self}")


@dataclass
class MoePlan:
    coef: torch.Tensor         # (T, top) float32 weights of the chosen
    idx: torch.Tensor          # (T, top) int32 chosen experts
    order: torch.Tensor        # (T * top,) pairs, expert by expert
    tiles: torch.Tensor        # (n, 4) expert, first slot, slots
    how: int                   # kernel of the grouped products


def moe_plan(z: torch.Tensor, bias: Optional[torch.Tensor],
             routing: Union[int, Routing], how: int) -> MoePlan:
    """Choose the experts of every row from its logits z (plainly, if
    ``routing`` is just their number), and group the pairs."""
    T, E = z.shape
    if isinstance(routing, int):
        routing = Routing(routing)
    assert z.dtype == torch.float32 and z.is_contiguous() and z.is_cuda
    routing.check(E)
    top = routing.top
    pairs, rows = T * top, MOE_TILE_ROWS[how]
    n = min(pairs, pairs // rows + E)
    ints = torch.empty(2 * pairs + 4 * n, dtype=torch.int32, device=z.device)
    p = MoePlan(torch.empty(T, top, dtype=torch.float32, device=z.device),
                ints[4 * n:4 * n + pairs].view(T, top), ints[4 * n + pairs:],
                ints[:4 * n].view(n, 4), how)
    a = _MoePlanArgs(z=_p(z), bias=_p(bias), idx=_p(p.idx), coef=_p(p.coef),
                     order=_p(p.order), tiles=_p(p.tiles), T=T, E=E, top=top,
                     tile_rows=rows, max_tiles=n,
                     kind=routing.kind, groups=routing.groups,
                     keep=routing.keep, best=routing.best)
    _check(library().sv_moe_plan(
        ctypes.byref(a), 0 if bias is None else _f32(bias), _stream()),
        "moe_plan")
    return p


def moe_gemm(x: torch.Tensor, w: torch.Tensor, plan: MoePlan, gated: bool,
             alpha: float = 1.0, limit: float = float("inf"),
             shift: float = 0.0) -> torch.Tensor:
    """Grouped product over w (E, rows, K).  ``gated``: rows of x (T, K) ->
    min(g, limit) sigmoid(alpha g) (clamp(u, limit) + shift) of w = [gate;
    up], in slot order.  Else: slots x (T * top, K) -> pairs."""
    pairs = plan.order.shape[0]
    N, K = w.shape[1] // (2 if gated else 1), w.shape[2]
    assert x.stride(1) == 1 and x.shape[1] == K and w.is_contiguous()
    assert x.dtype == w.dtype and w.shape[1] == N * (2 if gated else 1)
    assert x.shape[0] == (plan.coef.shape[0] if gated else pairs)
    out = torch.empty(pairs, N, dtype=x.dtype, device=x.device)
    a = _MoeGemmArgs(x=_p(x), xst=x.stride(0), w=_p(w), out=_p(out),
                     order=_p(plan.order), tiles=_p(plan.tiles),
                     top=plan.coef.shape[1] if gated else 0, N=N, K=K,
                     max_tiles=plan.tiles.shape[0], alpha=alpha, limit=limit,
                     shift=shift)
    assert plan.how == MOE_PLAIN or (x.dtype == torch.bfloat16
                                     and _aligned((N, K), x))
    _check(library().sv_moe_gemm(ctypes.byref(a), plan.how, int(gated),
                                 _f32(x), _stream()), "moe_gemm")
    return out


def moe_mlp(h, z, bias, gate_up, down, routing: Union[int, Routing],
            alpha: float, limit: float, shift: float) -> Pending:
    """Gated experts on h (T, W) with router logits z (T, E): a pending sum
    of the chosen experts' outputs."""
    if isinstance(routing, int):
        routing = Routing(routing)
    E, W, ff = down.shape
    pairs = h.shape[0] * routing.top
    fast = h.dtype == torch.bfloat16 and _aligned((W, ff), h)
    plan = moe_plan(z, bias, routing,
                    moe_kernel(pairs, E) if fast else MOE_PLAIN)
    act = moe_gemm(h, gate_up, plan, True, alpha, limit, shift)
    return Pending(moe_gemm(act, down, plan, False), coef=plan.coef)
