// Recurrent matrix-memory mixers for ragged batches.
//
//   S_t = a_t S_(t-1) + b_t k_t v_t^T,    o_t = S_t^T q_t
//
// per head, with a 32-bit state S [D][E] per (slot, head) that lives across
// steps.  Two gatings share the kernels:
//
//   decay  a_t = decay_h, b_t = 1; q, k and v pass through silu.
//   gated  log gates i, f from a projection, soft-capped:
//            i = cap tanh(x_i / cap), f = logsigmoid(cap tanh(x_f / cap)),
//          a running maximum m keeps S and the normaliser n in range:
//            m_t = max(f + m_(t-1), i), a_t = exp(f + m_(t-1) - m_t),
//            b_t = exp(i - m_t), n_t = a_t n_(t-1) + b_t k_t,
//            o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6);
//          q is scaled by qscale.  S, n and m are zero at position 0.
//
//   sv_memory_steps   token after token; single-token decoding, the 32-bit
//                     mode and sizes the chunk kernel does not take
//   sv_memory_chunks  64-token chunks on MFMA for bf16 prompt portions
//
// Every group of 32 state columns keeps its own copy of n and m, so the
// workgroups of a head never wait for each other.
//
// A segment whose context is empty starts from zero instead of reading its
// slot, so a slot needs no clearing when it changes hands.

#include "serving.h"

#define GATED_EPS 1e-6f

struct MemoryArgs {
  const void *q, *k, *v;    // first row of the step's projections
  long qst, kst, vst;       // row strides (elements)
  const float* gates;       // [T][2 H] raw i then f (gated)
  const void *ib, *fb;      // [H] gate biases, T (gated)
  const float* decay;       // [H] (decay)
  const float* log2_decay;  // [H] (decay)
  float* S;                 // [slots][H][D][E]
  float* n;                 // [slots][H][ceil(E / 32)][D] (gated)
  float* m;                 // [slots][H][ceil(E / 32)] (gated)
  const int* seg;           // [n_seg][4]: slot, first row, rows, context
  void* out;                // [T][H * E]
  int H, D, E;
  float gate_cap, qscale;
};

__device__ __forceinline__ void log_gates(const MemoryArgs& a, long row,
                                          int h, float ib, float fb,
                                          float& i, float& f) {
  const float* g = a.gates + row * 2 * a.H;
  i = a.gate_cap * tanhf((g[h] + ib) / a.gate_cap);
  f = log_sigmoid_f(a.gate_cap * tanhf((g[a.H + h] + fb) / a.gate_cap));
}

// ---------------------------------------------------------------------------
// token after token: a workgroup owns 32 columns of one head's state
// ---------------------------------------------------------------------------
template <typename T, int NI, bool GATED, bool VEC>
__global__ void __launch_bounds__(256)
memory_steps_kernel(MemoryArgs a) {
  const int D = a.D, E = a.E;
  const int nt = (E + 31) / 32;
  const int vt = blockIdx.x % nt;
  const int h = blockIdx.x / nt % a.H;
  const int* sg = a.seg + 4 * (blockIdx.x / nt / a.H);
  const long slot = sg[0];
  const int row0 = sg[1], nrow = sg[2], ctx = sg[3];
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int vq = tid & 7, dg = tid >> 3;
  const int e0 = vt * 32 + 4 * vq;

  __shared__ float sq[2][NI * 32], sk[2][NI * 32], sv[2][32];
  __shared__ float red[2][4][32], redn[2][4];

  float* Sp = a.S + (slot * a.H + h) * D * E;
  float S[NI][4];
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int d = dg + 32 * i;
#pragma unroll
    for (int j = 0; j < 4; ++j) S[i][j] = 0.f;
    if (ctx > 0 && d < D) {
      if (VEC) {
        if (e0 < E) load4(Sp + (long)d * E + e0, S[i]);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (e0 + j < E) S[i][j] = Sp[(long)d * E + e0 + j];
      }
    }
  }
  // n: dim d belongs to thread d (and d + 256)
  constexpr int NN = (NI * 32 + 255) / 256;
  float n[NN], m = 0.f, ib = 0.f, fb = 0.f;
  if (GATED) {
#pragma unroll
    for (int i = 0; i < NN; ++i) {
      const int d = tid + 256 * i;
      n[i] = ctx > 0 && d < D ? a.n[((slot * a.H + h) * nt + vt) * D + d] : 0.f;
    }
    if (ctx > 0) m = a.m[(slot * a.H + h) * nt + vt];
    ib = to_f(((const T*)a.ib)[h]);
    fb = to_f(((const T*)a.fb)[h]);
  }
  const float decay = GATED ? 0.f : a.decay[h];

  for (int t = 0; t < nrow; ++t) {
    const long row = row0 + t;
    const int b = t & 1;
    for (int d = tid; d < NI * 32; d += 256) {
      float x = 0.f, y = 0.f;
      if (d < D) {
        x = to_f(((const T*)a.q)[row * a.qst + (long)h * D + d]);
        y = to_f(((const T*)a.k)[row * a.kst + (long)h * D + d]);
        if (GATED) x *= a.qscale;
        else { x = silu_f(x); y = silu_f(y); }
      }
      sq[b][d] = x;
      sk[b][d] = y;
    }
    if (tid < 32) {
      const int e = vt * 32 + tid;
      float x = e < E ? to_f(((const T*)a.v)[row * a.vst + (long)h * E + e])
                      : 0.f;
      sv[b][tid] = GATED ? x : silu_f(x);
    }
    float fs = decay, is = 1.f;
    if (GATED) {
      float gi, gf;
      log_gates(a, row, h, ib, fb, gi, gf);
      const float mn = fmaxf(gf + m, gi);
      fs = expf(gf + m - mn);
      is = expf(gi - mn);
      m = mn;
    }
    __syncthreads();
    float v[4], o[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = sv[b][4 * vq + j] * is;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const float kd = sk[b][dg + 32 * i], qd = sq[b][dg + 32 * i];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        S[i][j] = fs * S[i][j] + kd * v[j];
        o[j] += qd * S[i][j];
      }
    }
#pragma unroll
    for (int off = 8; off < 64; off <<= 1)
#pragma unroll
      for (int j = 0; j < 4; ++j) o[j] += __shfl_xor(o[j], off, 64);
    if (lane < 8)
#pragma unroll
      for (int j = 0; j < 4; ++j) red[b][wid][4 * vq + j] = o[j];
    if (GATED) {
      float nq = 0.f;
#pragma unroll
      for (int i = 0; i < NN; ++i) {
        const int d = tid + 256 * i;
        if (d < NI * 32) {
          n[i] = fs * n[i] + is * sk[b][d];
          nq += n[i] * sq[b][d];
        }
      }
      nq = wave_reduce(nq, SumOp());
      if (lane == 0) redn[b][wid] = nq;
    }
    __syncthreads();
    if (tid < 32 && vt * 32 + tid < E) {
      float r = red[b][0][tid] + red[b][1][tid] + red[b][2][tid] +
                red[b][3][tid];
      if (GATED) {
        const float nq = redn[b][0] + redn[b][1] + redn[b][2] + redn[b][3];
        r /= fmaxf(fabsf(nq), expf(-m)) + GATED_EPS;
      }
      from_f(((T*)a.out)[row * a.H * E + (long)h * E + vt * 32 + tid], r);
    }
  }

#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int d = dg + 32 * i;
    if (d >= D) continue;
    if (VEC) {
      if (e0 < E) store4(Sp + (long)d * E + e0, S[i]);
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (e0 + j < E) Sp[(long)d * E + e0 + j] = S[i][j];
    }
  }
  if (GATED) {
#pragma unroll
    for (int i = 0; i < NN; ++i) {
      const int d = tid + 256 * i;
      if (d < D) a.n[((slot * a.H + h) * nt + vt) * D + d] = n[i];
    }
    if (tid == 0) a.m[(slot * a.H + h) * nt + vt] = m;
  }
}

template <typename T, bool GATED>
static int launch_steps(const MemoryArgs& a, int n_seg, hipStream_t stream) {
  const long grid = (long)n_seg * a.H * ((a.E + 31) / 32);
  const bool vec = a.E % 4 == 0;
#define MS(N, V) memory_steps_kernel<T, N, GATED, V><<<grid, 256, 0, stream>>>(a)
#define MSV(N) do { if (vec) MS(N, true); else MS(N, false); } while (0)
  if (a.D <= 64) MSV(2);
  else if (a.D <= 128) MSV(4);
  else if (a.D <= 256) MSV(8);
  else if (a.D <= 512) MSV(16);
  else return 1;
#undef MSV
#undef MS
  return (int)hipGetLastError();
}

extern "C" int sv_memory_steps(const MemoryArgs* a, int n_seg, int gated,
                               int f32, hipStream_t stream) {
  if (n_seg <= 0) return 0;
  if (f32)
    return gated ? launch_steps<float, true>(*a, n_seg, stream)
                 : launch_steps<float, false>(*a, n_seg, stream);
  return gated ? launch_steps<short, true>(*a, n_seg, stream)
               : launch_steps<short, false>(*a, n_seg, stream);
}

// ---------------------------------------------------------------------------
// 64-token chunks on MFMA (bf16 projections, 32-bit everything else)
//
// A workgroup (4 waves) carries VT columns of one head's state through the
// chunks of a segment; the state stays in MFMA accumulators.  With the local
// cumulative log forget b_t and a_s = i_s - b_s, M_t = max(m, max_{s<=t} a_s):
//
//   o_t = e^(m - M_t) S^T q_t + sum_{s<=t} e^(a_s - M_t) (q_t . k_s) v_s
//   S'  = e^(m - M_C) S + sum_s e^(a_s - M_C) k_s v_s^T,  m' = b_C + M_C
//
// (every exponent is <= 0).  The plain decay is the same with
// e^(a_s - M_t) -> decay^(t-s).
//
// 32-bit operands meet bf16 ones exactly: an f32 value is split into three
// bf16 planes (8 + 8 + 8 bits) and each plane is multiplied on its own.
// Products are 16x16x32; a wave owns 16 query rows.  Scores are produced
// transposed (lane = query), so they feed the next product as its B operand
// without leaving registers: the contraction order is the accumulator's row
// order, and V^T is read from LDS in that same order.
// ---------------------------------------------------------------------------
__device__ __forceinline__ f32x4 mfma16(const frag_u& a, const frag_u& b,
                                        f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.bf, b.bf, c, 0, 0, 0);
}

// split a pair of floats into three planes of packed bf16
__device__ __forceinline__ void split3(float x, float y, uint* w) {
#pragma unroll
  for (int z = 0; z < 3; ++z) {
    w[z] = pack_bf16x2(x, y);
    x -= __uint_as_float(w[z] << 16);
    y -= __uint_as_float(w[z] & 0xffff0000u);
  }
}

__device__ __forceinline__ void unpack8(uint4v u, float* v) {
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    v[2 * j] = __uint_as_float(u[j] << 16);
    v[2 * j + 1] = __uint_as_float(u[j] & 0xffff0000u);
  }
}
__device__ __forceinline__ uint4v silu8(uint4v u) {
  float v[8];
  unpack8(u, v);
#pragma unroll
  for (int j = 0; j < 4; ++j)
    u[j] = pack_bf16x2(silu_f(v[2 * j]), silu_f(v[2 * j + 1]));
  return u;
}

template <int DP, bool GATED>
__global__ void __launch_bounds__(256)
memory_chunks_kernel(MemoryArgs a) {
  constexpr int VT = 32;
  constexpr int NK = DP / 32;          // 32-deep steps over the key size
  constexpr int MT = DP / 64;          // 16-row state tiles of a wave
  constexpr int KB = DP * 2 + 16;      // K row pitch (bytes)
  constexpr int TP = 72;               // pitch of s-contiguous rows
  constexpr int SP = DP + 8;           // S^T plane pitch (elements)
  constexpr int CPR = DP / 8;
  constexpr int PAIRS = 32 * CPR / 256;
  __shared__ __attribute__((aligned(16))) char kbuf[64 * KB];
  __shared__ __attribute__((aligned(16))) short ktb[DP * TP];
  __shared__ __attribute__((aligned(16))) short vtb[VT * TP];
  __shared__ __attribute__((aligned(16))) short vwb[3][VT * TP];
  __shared__ __attribute__((aligned(16))) short spl[3][VT * SP];
  __shared__ float s_a[64], s_M[64], s_in[64], s_w[64], s_em[64];
  __shared__ float s_n[DP];
  __shared__ float s_m[2];             // m, and the state factor of a chunk

  const int D = a.D, E = a.E;
  const int nt = (E + VT - 1) / VT;
  const int vt = blockIdx.x % nt;
  const int h = blockIdx.x / nt % a.H;
  const int* sg = a.seg + 4 * (blockIdx.x / nt / a.H);
  const long slot = sg[0];
  const int row0 = sg[1], nrow = sg[2], ctx = sg[3];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int c16 = lane & 15, g = lane >> 4;
  const int e0 = vt * VT;

  const short* qp = (const short*)a.q + (long)h * D;
  const short* kp = (const short*)a.k + (long)h * D;
  const short* vp = (const short*)a.v + (long)h * E + e0;
  const float l2d = GATED ? 0.f : a.log2_decay[h];

  // state: lane holds S[d = 16 (wid MT + i) + 4 g + r][e0 + 16 j + c16]
  float* Sp = a.S + (slot * a.H + h) * D * E;
  f32x4 S[MT][2] = {};
  if (ctx > 0) {
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int d = 16 * (wid * MT + i) + 4 * g + r;
          const int e = e0 + 16 * j + c16;
          if (d < D && e < E) S[i][j][r] = Sp[(long)d * E + e];
        }
  }
  float ib = 0.f, fb = 0.f;
  if (GATED) {
    for (int d = tid; d < DP; d += 256)
      s_n[d] = ctx > 0 && d < D ? a.n[((slot * a.H + h) * nt + vt) * D + d] : 0.f;
    if (tid == 0) s_m[0] = ctx > 0 ? a.m[(slot * a.H + h) * nt + vt] : 0.f;
    ib = bits2f(((const short*)a.ib)[h]);
    fb = bits2f(((const short*)a.fb)[h]);
  }

  // the next chunk's rows travel in registers while this one is computed
  uint4v kreg[2 * PAIRS], vreg[2];
  frag_u qreg[NK];
  float gi = 0.f, gf = 0.f;
  const int v_r = tid >> 2 << 1, v_c = (tid & 3) * 8;  // tid < 128
  auto issue = [&](int c0) {
    const int L = min(64, nrow - c0);
    const uint4v zero = {0, 0, 0, 0};
#pragma unroll
    for (int p = 0; p < PAIRS; ++p) {
      const int it = p * 256 + tid;
      const int r = it / CPR * 2, c = it % CPR * 8;
#pragma unroll
      for (int x = 0; x < 2; ++x)
        kreg[2 * p + x] = r + x < L && c < D
            ? *(const uint4v*)(kp + (row0 + c0 + r + x) * a.kst + c) : zero;
    }
    if (tid < 128) {
#pragma unroll
      for (int x = 0; x < 2; ++x)
        vreg[x] = v_r + x < L && e0 + v_c < E
            ? *(const uint4v*)(vp + (row0 + c0 + v_r + x) * a.vst + v_c)
            : zero;
    }
    const int t = 16 * wid + c16;
#pragma unroll
    for (int s = 0; s < NK; ++s) {
      const int d = 32 * s + 8 * g;
      qreg[s].u4 = t < L && d < D
          ? *(const uint4v*)(qp + (row0 + c0 + t) * a.qst + d) : zero;
    }
    if (GATED && wid == 0) {
      gi = gf = 0.f;
      if (lane < L) {
        const float* gr = a.gates + (long)(row0 + c0 + lane) * 2 * a.H;
        gi = gr[h];
        gf = gr[a.H + h];
      }
    }
  };

  issue(0);
  for (int c0 = 0; c0 < nrow; c0 += 64) {
    const int L = min(64, nrow - c0);
    __syncthreads();                     // LDS of the previous chunk is free

    // ---- gates / decay weights of the chunk (wave 0, lane = token) -------
    if (wid == 0) {
      if (GATED) {
        float i = -INFINITY, f = 0.f;
        if (lane < L) {
          i = a.gate_cap * tanhf((gi + ib) / a.gate_cap);
          f = log_sigmoid_f(a.gate_cap * tanhf((gf + fb) / a.gate_cap));
        }
        float b = f;
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
          const float o = __shfl_up(b, off, 64);
          if (lane >= off) b += o;
        }
        const float as = i - b;
        float M = as;
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
          const float o = __shfl_up(M, off, 64);
          if (lane >= off) M = fmaxf(M, o);
        }
        const float m0 = s_m[0];
        M = fmaxf(M, m0);
        const float Mc = __shfl(M, 63, 64), bc = __shfl(b, 63, 64);
        s_a[lane] = as;
        s_M[lane] = M;
        s_in[lane] = expf(m0 - M);
        s_w[lane] = expf(as - Mc);       // 0 past the end (as = -inf)
        s_em[lane] = expf(-(b + M));
        if (lane == 63) {
          s_m[1] = expf(m0 - Mc);
          s_m[0] = bc + Mc;
        }
      } else {
        s_in[lane] = __builtin_amdgcn_exp2f((lane + 1) * l2d);
        s_w[lane] = lane < L ? (lane == L - 1 ? 1.f
            : __builtin_amdgcn_exp2f((L - 1 - lane) * l2d)) : 0.f;
        if (lane == 0) s_m[1] = __builtin_amdgcn_exp2f(L * l2d);
      }
    }
    // ---- stage K, K^T, and the state's planes ----------------------------
    frag_u qf[NK];
#pragma unroll
    for (int s = 0; s < NK; ++s)
      qf[s].u4 = GATED ? qreg[s].u4 : silu8(qreg[s].u4);
#pragma unroll
    for (int p = 0; p < PAIRS; ++p) {
      const int it = p * 256 + tid;
      const int r = it / CPR * 2, c = it % CPR * 8;
      union { uint4v u; unsigned short s[8]; } x, y;
      x.u = GATED ? kreg[2 * p] : silu8(kreg[2 * p]);
      y.u = GATED ? kreg[2 * p + 1] : silu8(kreg[2 * p + 1]);
      *(uint4v*)(kbuf + r * KB + c * 2) = x.u;
      *(uint4v*)(kbuf + (r + 1) * KB + c * 2) = y.u;
#pragma unroll
      for (int j = 0; j < 8; ++j)
        *(uint*)(ktb + (c + j) * TP + r) = (uint)x.s[j] | ((uint)y.s[j] << 16);
    }
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        uint w0[3], w1[3];
        split3(S[i][j][0], S[i][j][1], w0);
        split3(S[i][j][2], S[i][j][3], w1);
        const int off =
            (16 * j + c16) * SP + 16 * (wid * MT + i) + 4 * g;
#pragma unroll
        for (int z = 0; z < 3; ++z)
          *(uint2*)(&spl[z][off]) = uint2{w0[z], w1[z]};
      }
    __syncthreads();                     // weights are visible

    // ---- stage V^T and the weighted V planes -----------------------------
    if (tid < 128) {
      const uint4v x = GATED ? vreg[0] : silu8(vreg[0]);
      const uint4v y = GATED ? vreg[1] : silu8(vreg[1]);
      float xf[8], yf[8];
      unpack8(x, xf);
      unpack8(y, yf);
      const float wx = s_w[v_r], wy = s_w[v_r + 1];
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        uint w[3];
        split3(xf[j] * wx, yf[j] * wy, w);
        const int off = (v_c + j) * TP + v_r;
        *(uint*)(vtb + off) = pack_bf16x2(xf[j], yf[j]);
#pragma unroll
        for (int z = 0; z < 3; ++z) *(uint*)(&vwb[z][off]) = w[z];
      }
    }
    if (c0 + 64 < nrow) issue(c0 + 64);

    // ---- scores^T of this wave's 16 queries against s <= t ---------------
    const int t = 16 * wid + c16;
    f32x4 P[4] = {};
#pragma unroll
    for (int st = 0; st < 4; ++st) {
      if (st > wid) continue;            // wave-uniform
#pragma unroll
      for (int s = 0; s < NK; ++s) {
        frag_u kf;
        kf.u4 = *(const uint4v*)(kbuf + (16 * st + c16) * KB +
                                 (32 * s + 8 * g) * 2);
        P[st] = mfma16(kf, qf[s], P[st]);
      }
    }
    const float qs = GATED ? a.qscale : 1.f;
    const float Mt = GATED ? s_M[t] : 0.f;
    float rowsum = 0.f;
#pragma unroll
    for (int st = 0; st < 4; ++st)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int s = 16 * st + 4 * g + r;
        float w = 0.f;
        if (s <= t && st <= wid) {
          if (GATED) w = __expf(s_a[s] - Mt) * qs;
          else w = s == t ? 1.f : __builtin_amdgcn_exp2f((t - s) * l2d);
        }
        P[st][r] *= w;
        rowsum += P[st][r];
      }

    // ---- the carried state's part ----------------------------------------
    f32x4 O[2] = {};
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int z = 0; z < 3; ++z)
#pragma unroll
        for (int s = 0; s < NK; ++s) {
          frag_u sf;
          sf.u4 = *(const uint4v*)(&spl[z][(16 * j + c16) * SP + 32 * s +
                                           8 * g]);
          O[j] = mfma16(sf, qf[s], O[j]);
        }
    const float in = s_in[t] * qs;
    O[0] *= in;
    O[1] *= in;
    float den = 1.f;
    if (GATED) {
      float nq = 0.f;
#pragma unroll
      for (int s = 0; s < NK; ++s) {
        float qv[8];
        unpack8(qf[s].u4, qv);
#pragma unroll
        for (int j = 0; j < 8; ++j) nq += qv[j] * s_n[32 * s + 8 * g + j];
      }
      float d = rowsum + nq * in;
      d += __shfl_xor(d, 16, 64);
      d += __shfl_xor(d, 32, 64);
      den = 1.f / (fmaxf(fabsf(d), s_em[t]) + GATED_EPS);
    }
    __syncthreads();                     // V^T is staged; s_n was read

    // ---- the chunk's own part --------------------------------------------
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      if (2 * kk > wid) continue;
      frag_u pf[3];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const f32x4& p = P[2 * kk + (u >> 1)];
        uint w[3];
        split3(p[2 * (u & 1)], p[2 * (u & 1) + 1], w);
#pragma unroll
        for (int z = 0; z < 3; ++z) pf[z].u[u] = w[z];
      }
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const short* vr = vtb + (16 * j + c16) * TP + 32 * kk + 4 * g;
        frag_u vf;
        *(uint2*)&vf.u[0] = *(const uint2*)vr;
        *(uint2*)&vf.u[2] = *(const uint2*)(vr + 16);
#pragma unroll
        for (int z = 0; z < 3; ++z) O[j] = mfma16(vf, pf[z], O[j]);
      }
    }
    if (t < L) {
      short* dst = (short*)a.out + ((long)(row0 + c0 + t) * a.H + h) * E + e0;
#pragma unroll
      for (int j = 0; j < 2; ++j)
        if (e0 + 16 * j + 4 * g < E)
          *(uint2*)(dst + 16 * j + 4 * g) =
              uint2{pack_bf16x2(O[j][0] * den, O[j][1] * den),
                    pack_bf16x2(O[j][2] * den, O[j][3] * den)};
    }

    // ---- advance the state -----------------------------------------------
    const float fac = s_m[1];
#pragma unroll
    for (int i = 0; i < MT; ++i) {
      frag_u kf[2];
#pragma unroll
      for (int kk = 0; kk < 2; ++kk)
        kf[kk].u4 = *(const uint4v*)(ktb + (16 * (wid * MT + i) + c16) * TP +
                                     32 * kk + 8 * g);
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        S[i][j] *= fac;
#pragma unroll
        for (int z = 0; z < 3; ++z)
#pragma unroll
          for (int kk = 0; kk < 2; ++kk) {
            frag_u vf;
            vf.u4 = *(const uint4v*)(&vwb[z][(16 * j + c16) * TP + 32 * kk +
                                             8 * g]);
            S[i][j] = mfma16(kf[kk], vf, S[i][j]);
          }
      }
    }
    if (GATED) {
      for (int d = tid; d < DP; d += 256) {
        float n = fac * s_n[d];
#pragma unroll
        for (int s = 0; s < 64; s += 8) {
          float kv[8];
          unpack8(*(const uint4v*)(ktb + d * TP + s), kv);
#pragma unroll
          for (int j = 0; j < 8; ++j) n += s_w[s + j] * kv[j];
        }
        s_n[d] = n;
      }
    }
  }

#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = 16 * (wid * MT + i) + 4 * g + r;
        const int e = e0 + 16 * j + c16;
        if (d < D && e < E) Sp[(long)d * E + e] = S[i][j][r];
      }
  if (GATED) {
    for (int d = tid; d < D; d += 256)
      a.n[((slot * a.H + h) * nt + vt) * D + d] = s_n[d];
    if (tid == 0) a.m[(slot * a.H + h) * nt + vt] = s_m[0];
  }
}

// bf16; D and E multiples of 8 with D <= 256; 16-byte aligned rows
extern "C" int sv_memory_chunks(const MemoryArgs* a, int n_seg, int gated,
                                hipStream_t stream) {
  if (n_seg <= 0) return 0;
  const long grid = (long)n_seg * a->H * ((a->E + 31) / 32);
#define MC(P)                                                              \
  do {                                                                     \
    if (gated) memory_chunks_kernel<P, true><<<grid, 256, 0, stream>>>(*a); \
    else memory_chunks_kernel<P, false><<<grid, 256, 0, stream>>>(*a);      \
  } while (0)
  if (a->D <= 64) MC(64);
  else if (a->D <= 128) MC(128);
  else if (a->D <= 256) MC(256);
  else return 1;
#undef MC
  return (int)hipGetLastError();
}
