"""Serving kernels: ragged batches over a paged KV cache and state slots.

Python wrappers of ``libnxd_serving.so`` (``csrc/serving/*.hip``).  They run
on the GPU only — there is no eager substitute, a CPU tensor or a missing
library raises.  Activations and weights are bfloat16, or float32 in the
32-bit mode; the residual stream, attention scores and weights, norms,
gates and recurrent state are 32-bit in both.
"""

import ctypes
import os
from dataclasses import dataclass
from typing import Optional

import torch

PAGE_SIZE = 64
MAX_HEAD_DIM = 512          # attention q/k and v size, recurrent q/k size
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


class _ResidualNormArgs(ctypes.Structure):
    _fields_ = (_fields("x delta delta2 w1 w2 vec x_out h w cat x0 index",
                        ctypes.c_void_p)
                + _fields("rows_out W delta_f32", ctypes.c_int)
                + _fields("eps branch_scale", ctypes.c_float))


class _RowsArgs(ctypes.Structure):
    _fields_ = (_fields("q k v", ctypes.c_void_p)
                + _fields("qst kst vst", ctypes.c_long)
                + _fields("kc vc pos seq bt part out", ctypes.c_void_p)
                + _fields("MB rows H G D E splits append window keep",
                          ctypes.c_int)
                + _fields("scale", ctypes.c_float))


class _TilesArgs(ctypes.Structure):
    _fields_ = (_fields("q", ctypes.c_void_p) + _fields("qst", ctypes.c_long)
                + _fields("kc vc tiles bt out", ctypes.c_void_p)
                + _fields("MB H G D E window keep", ctypes.c_int)
                + _fields("scale", ctypes.c_float))


class _MemoryArgs(ctypes.Structure):
    _fields_ = (_fields("q k v", ctypes.c_void_p)
                + _fields("qst kst vst", ctypes.c_long)
                + _fields("gates ib fb decay log2_decay S n m seg out",
                          ctypes.c_void_p)
                + _fields("H D E", ctypes.c_int)
                + _fields("gate_cap qscale", ctypes.c_float))


class _ChunkArgs(ctypes.Structure):
    _fields_ = ([("a", _MemoryArgs)] + _fields("chunks first", ctypes.c_void_p)
                + _fields("n_chunks n_seg T", ctypes.c_int)
                + _fields("b i c tot cend U N P mst VT KA", ctypes.c_void_p))


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
    tensor, or two branches that are RMS-normed with their own weights,
    scaled and summed.  ``vec`` is a row added to every token."""
    delta: torch.Tensor
    delta2: Optional[torch.Tensor] = None
    w1: Optional[torch.Tensor] = None
    w2: Optional[torch.Tensor] = None
    branch_scale: float = 1.0
    vec: Optional[torch.Tensor] = None


def residual_norm(x: Optional[torch.Tensor], pending: Optional[Pending],
                  eps: float, weight: Optional[torch.Tensor] = None,
                  x0: Optional[torch.Tensor] = None, keep_x: bool = True,
                  index: Optional[torch.Tensor] = None, dtype=None):
    """Add ``pending`` to the float32 residual ``x`` (None: zero) and return
    (new x or None, RMS-normed row * weight or None, [new x; x0] or None)."""
    src = x if pending is None else pending.delta
    rows, W = src.shape
    dtype = dtype or (weight if weight is not None else x0).dtype
    f32 = _f32(src) if dtype == torch.float32 else 0
    out_rows = rows if index is None else index.shape[0]
    dev = src.device
    x_new = torch.empty(out_rows, W, dtype=torch.float32, device=dev) \
        if keep_x else None
    h = torch.empty(out_rows, W, dtype=dtype, device=dev) \
        if weight is not None else None
    cat = torch.empty(out_rows, 2 * W, dtype=dtype, device=dev) \
        if x0 is not None else None
    a = _ResidualNormArgs(rows_out=out_rows, W=W, eps=eps)
    a.x, a.x_out, a.h, a.w = _p(x), _p(x_new), _p(h), _p(weight)
    a.cat, a.x0, a.index = _p(cat), _p(x0), _p(index)
    if pending is not None:
        d = pending.delta
        assert d.is_contiguous() and d.dtype in (dtype, torch.float32)
        assert pending.delta2 is None or (
            d.dtype == dtype and pending.delta2.is_contiguous()
            and pending.delta2.shape == d.shape)
        a.delta, a.delta2 = _p(d), _p(pending.delta2)
        a.w1, a.w2, a.vec = _p(pending.w1), _p(pending.w2), _p(pending.vec)
        a.branch_scale = pending.branch_scale
        a.delta_f32 = int(d.dtype == torch.float32 and
                          dtype != torch.float32)
    _check(library().sv_residual_norm(ctypes.byref(a), f32, _stream()),
           "residual_norm")
    return x_new, h, cat


def gated_norm(o: torch.Tensor, weight: torch.Tensor, gate: torch.Tensor,
               group: int, eps: float) -> torch.Tensor:
    """o (T, N): every ``group`` elements divided by their root mean square,
    times weight (N,), times sigmoid(gate (T, N))."""
    T, N = o.shape
    assert N % group == 0 and gate.shape == o.shape
    assert gate.stride(1) == 1 and o.is_contiguous()
    out = torch.empty_like(o)
    vec4 = int(group % 4 == 0 and gate.stride(0) % 4 == 0
               and gate.storage_offset() % 4 == 0)
    _check(library().sv_gated_norm(
        ctypes.c_void_p(_p(o)), ctypes.c_void_p(_p(weight)),
        ctypes.c_void_p(_p(gate)), ctypes.c_long(gate.stride(0)),
        ctypes.c_void_p(_p(out)), T, N // group, group, ctypes.c_float(eps),
        vec4, _f32(o), _stream()), "gated_norm")
    return out


def relu_squared_(x: torch.Tensor) -> torch.Tensor:
    assert x.is_contiguous()
    _check(library().sv_relu_squared(ctypes.c_void_p(_p(x)),
                                     ctypes.c_long(x.numel()), _f32(x),
                                     _stream()), "relu_squared")
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


def attn_rows(q, k, v, kc, vc, pos, seq, block_table, heads: int,
              scale: float, window: int = 0, keep: int = 0,
              append: bool = True, max_keys: int = 0,
              out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """One query row per request row: decoding.  ``append`` also writes the
    row's own k/v into the cache (without it they must be there already).
    ``max_keys`` bounds the visible keys of any row (it only sets how many
    workgroups share a row)."""
    G, D, E = _check_cache(q, k, v, kc, vc, heads)
    rows = q.shape[0]
    assert pos.shape[0] == rows and seq.shape[0] == rows
    if window > 0:
        max_keys = min(max_keys, window + keep) if max_keys else window + keep
    want = max(1, 1024 // max(1, rows * G))
    splits = max(1, min(want, (max_keys + 127) // 128, 64))
    out = _out(out, rows, heads * E, q)
    part = torch.empty(rows * heads * splits * (E + 2), dtype=torch.float32,
                       device=q.device) if splits > 1 else None
    a = _RowsArgs(q=_p(q), k=_p(k), v=_p(v), qst=q.stride(0),
                  kst=k.stride(0), vst=v.stride(0), kc=_p(kc), vc=_p(vc),
                  pos=_p(pos), seq=_p(seq), bt=_p(block_table),
                  part=_p(part), out=_p(out), MB=block_table.shape[1],
                  rows=rows, H=heads, G=G, D=D, E=E, splits=splits,
                  append=int(append), window=window, keep=keep, scale=scale)
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
                  max_keys: int = 0,
                  out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Prompt portions: append k/v, then causal attention of every row over
    its request's cache.  ``tiles`` (n, 4) int32 lists (request, first row,
    rows <= 128, position of the first row)."""
    G, D, E = _check_cache(q, k, v, kc, vc, heads)
    kv_append(k, v, kc, vc, pos, seq, block_table)
    if not attn_tiles_supported(q, kc, vc):
        return attn_rows(q, k, v, kc, vc, pos, seq, block_table, heads,
                         scale, window, keep, append=False,
                         max_keys=max_keys, out=out)
    out = _out(out, q.shape[0], heads * E, q)
    a = _TilesArgs(q=_p(q), qst=q.stride(0), kc=_p(kc), vc=_p(vc),
                   tiles=_p(tiles), bt=_p(block_table), out=_p(out),
                   MB=block_table.shape[1], H=heads, G=G, D=D, E=E,
                   window=window, keep=keep, scale=scale)
    _check(library().sv_attn_tiles(ctypes.byref(a), tiles.shape[0],
                                   _stream()), "attn_tiles")
    return out


def ragged_attention(q, k, v, batch, pool, heads: int, scale: float,
                     window: int = 0, keep: int = 0) -> torch.Tensor:
    """Attention of a packed batch over its cache pool: portions first, then
    single tokens, into one (T, heads * E) tensor."""
    kc, vc = pool
    T, n = q.shape[0], batch.portion_tokens
    out = torch.empty(T, heads * vc.shape[3], dtype=q.dtype, device=q.device)
    args = dict(heads=heads, scale=scale, window=window, keep=keep,
                max_keys=batch.max_keys)
    if n:
        attn_portions(q[:n], k[:n], v[:n], kc, vc, batch.pos[:n],
                      batch.seq[:n], batch.block_table, batch.tiles,
                      out=out[:n], **args)
    if n < T:
        attn_rows(q[n:], k[n:], v[n:], kc, vc, batch.pos[n:], batch.seq[n:],
                  batch.block_table, out=out[n:], **args)
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
               out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Run a matrix memory over segments of a ragged batch.  q, k (T, H*D),
    v (T, H*E); S (slots, H, D, E) float32; n (slots, H, ceil(E/32), D) and
    m (slots, H, ceil(E/32)) float32 for an ExpGate.  ``seg`` (n, 4) int32
    lists (slot, first row, rows, context); rows count from the start of
    the tensors, so portions and single tokens of one batch can be run by
    two calls into one ``out``.  With the device form of
    ``chunk_table`` the 256-token MFMA kernels run where they apply."""
    D, E = S.shape[2], S.shape[3]
    T = q.shape[0]
    assert q.shape[1] == k.shape[1] == heads * D and v.shape[1] == heads * E
    assert q.stride(1) == k.stride(1) == v.stride(1) == 1
    assert S.is_contiguous() and S.dtype == torch.float32
    assert S.shape[1] == heads
    if D > MAX_HEAD_DIM:
        raise ValueError(f"key size {D} > {MAX_HEAD_DIM}")
    out = _out(out, T, heads * E, q)
    a = _MemoryArgs(q=_p(q), k=_p(k), v=_p(v), qst=q.stride(0),
                    kst=k.stride(0), vst=v.stride(0), S=_p(S), seg=_p(seg),
                    out=_p(out), H=heads, D=D, E=E, gate_cap=1.0, qscale=1.0)
    gated = isinstance(gate, ExpGate)
    if gated:
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
    lib = library()
    if (chunks is not None and q.dtype == torch.bfloat16 and D <= 256
            and _aligned((D, E), q, k, v)):
        nc = chunks.shape[0]
        assert chunk_first.shape[0] == seg.shape[0] + 1
        f32 = dict(dtype=torch.float32, device=q.device)
        U = torch.empty(nc, heads, E, D, **f32)
        P = torch.empty(nc, heads, 3, E, D, dtype=torch.bfloat16,
                        device=q.device)
        VT = torch.empty(nc, heads, E, CHUNK, dtype=torch.bfloat16,
                         device=q.device)
        KA = None if gated else torch.empty(T, heads * D, dtype=q.dtype,
                                            device=q.device)
        x = _ChunkArgs(a=a, chunks=_p(chunks), first=_p(chunk_first),
                       n_chunks=nc, n_seg=seg.shape[0], T=T, U=_p(U),
                       P=_p(P), VT=_p(VT), KA=_p(KA))
        if gated:
            bic = torch.empty(3, heads, T, **f32)
            small = torch.empty(nc, heads, 6 + D, **f32)
            x.b, x.i, x.c = (_p(t) for t in bic)
            flat, nh = small.view(-1), nc * heads
            x.tot, x.cend = _p(flat), _p(flat[4 * nh:])
            x.mst, x.N = _p(flat[5 * nh:]), _p(flat[6 * nh:])
        st = lib.sv_memory_chunks(ctypes.byref(x), int(gated), _stream())
    else:
        st = lib.sv_memory_steps(ctypes.byref(a), seg.shape[0], int(gated),
                                 _f32(q), _stream())
    _check(st, "memory_mix")
    return out


def decay_gate(decay, device) -> DecayGate:
    d = torch.tensor([float(x) for x in decay], dtype=torch.float64)
    # finite for a decay of zero: 0 tokens apart must still weigh 2^0
    log2 = torch.log2(d).clamp(min=-1e4)
    return DecayGate(d.float().to(device), log2.float().to(device))
