// Recurrent matrix-memory mixers for ragged batches.
//
//   S_t = a_t S_(t-1) + b_t k_t v_t^T,    o_t = S_t^T q_t
//
// per head, with a 32-bit state S [D][E] per (slot, head) that lives across
// steps.  Four gatings share the kernels:
//
//   decay  a_t = decay_h, b_t = 1; q, k and v pass through silu.
//   gated  log gates i, f from a projection, soft-capped:
//            i = cap tanh(x_i / cap), f = logsigmoid(cap tanh(x_f / cap)),
//          a running maximum m keeps S and the normaliser n in range:
//            m_t = max(f + m_(t-1), i), a_t = exp(f + m_(t-1) - m_t),
//            b_t = exp(i - m_t), n_t = a_t n_(t-1) + b_t k_t,
//            o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6);
//          q is scaled by qscale.  S, n and m are zero at position 0.
//   timed  a time step from a projection (state-space duality):
//            b_t = softplus(x + bias), a_t = exp(-exp(A_log) b_t),
//          heads share q and k in groups, o_t + skip v_t is multiplied by
//          silu(z).
//   turned a_t = decay_h, b_t = kscale; q and k are rotated at their position,
//          in halves: elements i and i + rot / 2 turn together.
//
//   sv_memory_steps   token after token; single-token decoding, the 32-bit
//                     mode and sizes the chunk kernels do not take
//   sv_memory_chunks  256-token chunks on MFMA for bf16 prompt portions
//
// Every group of 32 state columns keeps its own copy of n and m, so the
// workgroups of a head never wait for each other.
//
// A segment whose context is empty starts from zero instead of reading its
// slot, so a slot needs no clearing when it changes hands.

#include "serving.h"

#define GATED_EPS 1e-6f

enum Gating { DECAY = 0, GATED = 1, TIMED = 2, TURNED = 3 };

struct MemoryArgs {
  const void *q, *k, *v;    // first row of the step's projections
  long qst, kst, vst;       // row strides (elements)
  const float* gates;       // [T][2 H] raw i then f (gated); [T][H] (timed)
  const void *ib, *fb;      // [H] biases, T: of i and f (gated); of the time
                            //   step, and A_log (timed)
  const float* decay;       // [H] (decay, turned)
  const float* log2_decay;  // [H] (decay, turned)
  float* S;                 // [slots][H][D][E]
  float* n;                 // [slots][H][ceil(E / 32)][D] (gated)
  float* m;                 // [slots][H][ceil(E / 32)] (gated)
  const int* seg;           // [n_seg][4]: slot, first row, rows, context
  void* out;                // [T][H * E]
  int H, D, E;
  float gate_cap, qscale;
  // timed only
  int G;                    // heads of q and k
  const void* skip;         // [H], T
  const void* z;            // [T][H * E] rows
  long zst;
  // q, k and v of single tokens before their causal convolution (steps only)
  const void *cw, *cb;      // [taps][C], [C]; cw null: they have passed it
  void* ring;               // [slots][taps][C]: position p in place p % taps
  int taps, C, kch, qch;    // channels of v, k, q start at 0, kch, qch
  // turned only
  const double* freq;       // [rot / 2] radians a position
  int rot;
  float amp, kscale;        // cos and sin are multiplied by amp
};

__device__ __forceinline__ float softplus_f(float x) {
  return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x)));
}

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
// TAPS: 0 no convolution, 1 any number of taps, else this number
template <typename T, int NI, int GATE, bool VEC, int TAPS>
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
  if (GATE == GATED) {
#pragma unroll
    for (int i = 0; i < NN; ++i) {
      const int d = tid + 256 * i;
      n[i] = ctx > 0 && d < D ? a.n[((slot * a.H + h) * nt + vt) * D + d] : 0.f;
    }
    if (ctx > 0) m = a.m[(slot * a.H + h) * nt + vt];
  }
  constexpr bool fixed = GATE == DECAY || GATE == TURNED;
  if (!fixed) {
    ib = to_f(((const T*)a.ib)[h]);
    fb = to_f(((const T*)a.fb)[h]);
  }
  const float decay = fixed ? a.decay[h] : 0.f;
  const int hk = GATE == TIMED ? h / (a.H / a.G) : h;   // head of q and k
  constexpr bool conv = TAPS > 0;
  // The convolution of a single token: channel c's filter and earlier inputs,
  // and its result; `keep` writes the token's own input into the ring.
  constexpr int NT = TAPS > 1 ? TAPS : 1;
  const int last = (TAPS > 1 ? TAPS : a.taps) - 1;
  const int here = conv ? ctx % (last + 1) : 0;
  auto place = [&](int k) {              // of the input last - k tokens ago
    const int i = here - last + k;
    return (long)(i < 0 ? i + last + 1 : i) * a.C;
  };
  auto convolve = [&](float x, int c, bool keep) {
    T* ring = (T*)a.ring + slot * (last + 1) * a.C + c;
    const T* w = (const T*)a.cw + c;
    float y = to_f(((const T*)a.cb)[c]);
    if (TAPS > 1) {
      float f[NT], in[NT];
#pragma unroll
      for (int k = 0; k < NT; ++k) {
        f[k] = to_f(w[(long)k * a.C]);
        in[k] = k < NT - 1 ? to_f(ring[place(k)]) : x;
      }
#pragma unroll
      for (int k = 0; k < NT; ++k)
        y += k >= last - ctx ? f[k] * in[k] : 0.f;
    } else {
      for (int k = max(0, last - ctx); k < last; ++k)
        y += to_f(w[(long)k * a.C]) * to_f(ring[place(k)]);
      y += to_f(w[(long)last * a.C]) * x;
    }
    if (keep) from_f(ring[(long)here * a.C], x);
    return silu_f(y);
  };

  for (int t = 0; t < nrow; ++t) {
    const long row = row0 + t;
    const int b = t & 1;
    for (int d = tid; d < NI * 32; d += 256) {
      float x = 0.f, y = 0.f;
      if (d < D) {
        x = to_f(((const T*)a.q)[row * a.qst + (long)hk * D + d]);
        y = to_f(((const T*)a.k)[row * a.kst + (long)hk * D + d]);
        if (GATE == GATED) x *= a.qscale;
        if (GATE == TURNED && d < a.rot) {
          const int half = a.rot / 2;
          const bool low = d < half;
          const int i = low ? d : d - half;
          const long o = (long)hk * D + (low ? d + half : i);
          float c, s;
          turn(a.freq[i], ctx + t, &c, &s);
          c *= a.amp;
          s *= low ? -a.amp : a.amp;
          x = x * c + to_f(((const T*)a.q)[row * a.qst + o]) * s;
          y = y * c + to_f(((const T*)a.k)[row * a.kst + o]) * s;
        }
        if (GATE == TURNED) y *= a.kscale;
        if (GATE == DECAY) { x = silu_f(x); y = silu_f(y); }
        if (conv) {
          const bool keep = vt == 0 && h % (a.H / a.G) == 0;
          x = convolve(x, a.qch + hk * D + d, keep);
          y = convolve(y, a.kch + hk * D + d, keep);
        }
      }
      sq[b][d] = x;
      sk[b][d] = y;
    }
    if (tid < 32) {
      const int e = vt * 32 + tid;
      float x = e < E ? to_f(((const T*)a.v)[row * a.vst + (long)h * E + e])
                      : 0.f;
      if (GATE == DECAY) x = silu_f(x);
      if (conv && e < E) x = convolve(x, h * E + e, true);
      sv[b][tid] = x;
    }
    float fs = decay, is = 1.f;
    if (GATE == TIMED) {
      is = softplus_f(a.gates[row * a.H + h] + ib);
      fs = expf(-expf(fb) * is);
    }
    if (GATE == GATED) {
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
    if (GATE == GATED) {
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
      if (GATE == GATED) {
        const float nq = redn[b][0] + redn[b][1] + redn[b][2] + redn[b][3];
        r /= fmaxf(fabsf(nq), expf(-m)) + GATED_EPS;
      }
      if (GATE == TIMED) {
        const long at = (long)h * E + vt * 32 + tid;
        r += to_f(((const T*)a.skip)[h]) * sv[b][tid];
        r *= silu_f(to_f(((const T*)a.z)[row * a.zst + at]));
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
  if (GATE == GATED) {
#pragma unroll
    for (int i = 0; i < NN; ++i) {
      const int d = tid + 256 * i;
      if (d < D) a.n[((slot * a.H + h) * nt + vt) * D + d] = n[i];
    }
    if (tid == 0) a.m[(slot * a.H + h) * nt + vt] = m;
  }
}

template <typename T, int GATE, int TAPS>
static int launch_steps(const MemoryArgs& a, int n_seg, hipStream_t stream) {
  const long grid = (long)n_seg * a.H * ((a.E + 31) / 32);
  const bool vec = a.E % 4 == 0;
#define MS(N, V) memory_steps_kernel<T, N, GATE, V, TAPS><<<grid, 256, 0, stream>>>(a)
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

extern "C" int sv_memory_steps(const MemoryArgs* a, int n_seg, int gating,
                               int f32, hipStream_t stream) {
  if (n_seg <= 0) return 0;
#define MST(T, K) launch_steps<T, TIMED, K>(*a, n_seg, stream)
#define MS(T)                                                            \
  (gating == GATED   ? launch_steps<T, GATED, 0>(*a, n_seg, stream)      \
   : gating == DECAY ? launch_steps<T, DECAY, 0>(*a, n_seg, stream)      \
   : gating == TURNED ? launch_steps<T, TURNED, 0>(*a, n_seg, stream)    \
   : !a->cw ? MST(T, 0) : a->taps == 4 ? MST(T, 4) : MST(T, 1))
  if (gating == TURNED && (a->rot % 2 || a->rot > a->D)) return 1;
  return f32 ? MS(float) : MS(short);
#undef MS
#undef MST
}


// ---------------------------------------------------------------------------
// Chunks on MFMA (bf16 projections, 32-bit everything else)
//
// A portion is cut into chunks of 256 tokens, and every chunk is computed in
// parallel; only a scan over the chunks' states is sequential.  With local
// inclusive sums b_t of the log forgets, c_t = max(f_t + c_(t-1), i_t) from
// c = -inf, and m, S, n before the chunk:
//
//   gates    b_t, i_t, c_t of every token
//   states   U = sum_s e^(b_L - b_s + i_s - c_L) k_s v_s^T   (and N with k_s)
//   scan     m' = max(b_L + m, c_L)
//            S' = e^(b_L + m - m') S + e^(c_L - m') U        (n' likewise)
//   outputs  m_t = max(b_t + m, c_t)
//            o_t ~ e^(b_t + m - m_t) S^T q_t
//                  + sum_(s<=t) e^(b_t - b_s + i_s - m_t) (q_t . k_s) v_s
//
// every exponent is <= 0.  b is kept per 64 tokens (with the four totals of
// a chunk), so near tokens never cancel large sums.  The fixed decays have
// e^(b_t - b_s + i_s - m_t) = decay^(t-s) and no m; the timed gating has
// e^(b_t - b_s) times the time step of s, and no m.
//
// 32-bit operands meet bf16 ones exactly: an f32 value is split into three
// bf16 planes (8 + 8 + 8 bits) and each plane is multiplied on its own.
// Rotated queries and keys are split into two planes (a rest below 2^-17);
// where two split values meet, products below 2^-24 are left out.
// Scores are produced transposed (lane = query), so they feed the next
// product as its B operand from registers: the accumulator's row order is
// the contraction order, and V^T is read from LDS in that same order.
// ---------------------------------------------------------------------------
#define MC_L 256

struct ChunkArgs {
  MemoryArgs a;
  const int* chunks;        // [n_chunks][4]: segment, first row, rows, ctx > 0
                            //   or not the first chunk of its segment
  const int* first;         // [n_seg + 1] first chunk of a segment
  int n_chunks, n_seg, T;
  float *b, *i, *c;         // [H][T] (gated; timed: i is the step, no c)
  float *tot, *cend;        // [n_chunks][H][4], [n_chunks][H] (gated; timed:
                            //   no cend)
  float* U;                 // [n_chunks][H][E][D]
  float* N;                 // [n_chunks][H][D] (gated): N, then n before
  short* P;                 // [n_chunks][H][3][E][D] state before the chunk
  float* mst;               // [n_chunks][H] m before the chunk (gated)
  short* VT;                // [n_chunks][H][E][256] V^T, activated
  short* KA;                // [T][H][D] activated K (decay); two planes of
                            //   rotated K (turned)
  short* QA;                // two planes of rotated Q (turned)
  float norm_eps;           // turned, with z: every head over its root mean
                            //   square, times silu(z)
};

__host__ __device__ constexpr bool fixed_decay(int gate) {
  return gate == DECAY || gate == TURNED;
}
// planes of queries and keys
__host__ __device__ constexpr int qk_planes(int gate) {
  return gate == TURNED ? 2 : 1;
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
template <bool ON>
__device__ __forceinline__ uint4v silu8(uint4v u) {
  if (ON) {
    float v[8];
    unpack8(u, v);
#pragma unroll
    for (int j = 0; j < 4; ++j)
      u[j] = pack_bf16x2(silu_f(v[2 * j]), silu_f(v[2 * j + 1]));
  }
  return u;
}

// ---- gates: one block per (chunk, head), one thread per token -------------
template <int GATE>
__global__ void __launch_bounds__(MC_L)
memory_gates_kernel(ChunkArgs x) {
  const MemoryArgs& a = x.a;
  const int h = blockIdx.x % a.H, ch = blockIdx.x / a.H;
  const int row0 = x.chunks[4 * ch + 1], nrow = x.chunks[4 * ch + 2];
  const int t = threadIdx.x, lane = t & 63, wid = t >> 6;
  float i = -INFINITY, f = 0.f;
  const float ib = bits2f(((const short*)a.ib)[h]);
  const float fb = bits2f(((const short*)a.fb)[h]);
  if (t < nrow) {
    if (GATE == TIMED) {
      i = softplus_f(a.gates[(long)(row0 + t) * a.H + h] + ib);
      f = -expf(fb) * i;
    } else {
      log_gates(a, row0 + t, h, ib, fb, i, f);
    }
  }
  float F = f, I = i;                    // scan of (F, I) by (+, max)
#pragma unroll
  for (int off = 1; off < 64; off <<= 1) {
    const float F0 = __shfl_up(F, off, 64), I0 = __shfl_up(I, off, 64);
    if (lane >= off) {
      I = fmaxf(I0 + F, I);
      F += F0;
    }
  }
  __shared__ float sF[4], sI[4];
  if (lane == 63) {
    sF[wid] = F;
    sI[wid] = I;
  }
  __syncthreads();
  float c = -INFINITY;
  for (int w = 0; w < wid; ++w) c = fmaxf(c + sF[w], sI[w]);
  c = fmaxf(c + F, I);
  if (t < nrow) {
    const long o = (long)h * x.T + row0 + t;
    x.b[o] = F;
    x.i[o] = i;
    if (GATE == GATED) x.c[o] = c;
  }
  const long ci = (long)ch * a.H + h;
  if (lane == 63) x.tot[ci * 4 + wid] = F;
  if (GATE == GATED && t == MC_L - 1) x.cend[ci] = c;
}

// ---- rotation: one workgroup per token, q and k of all heads into planes ---
template <bool VEC>
__global__ void __launch_bounds__(256) memory_turn_kernel(ChunkArgs x) {
  extern __shared__ float cs[];          // cos [rot / 2], sin [rot / 2]
  const MemoryArgs& a = x.a;
  const int ch = blockIdx.x / MC_L, t = blockIdx.x % MC_L;
  if (t >= x.chunks[4 * ch + 2]) return;
  const long row = x.chunks[4 * ch + 1] + t;
  const int* sg = a.seg + 4L * x.chunks[4 * ch];
  const int p = sg[3] + (int)row - sg[1];
  const int half = a.rot / 2, D = a.D;
  for (int i = threadIdx.x; i < half; i += 256) {
    float c, s;
    turn(a.freq[i], p, &c, &s);
    cs[i] = c * a.amp;
    cs[half + i] = s * a.amp;
  }
  __syncthreads();
  const long HD = (long)a.H * D, plane = (long)x.T * HD;
  constexpr int V = VEC ? 8 : 1;
  const int items = (D - half) / V;      // of a head: pairs, then the rest
  auto get = [&](const short* s, float* v) {
    if (VEC) unpack8(*(const uint4v*)s, v); else v[0] = bits2f(s[0]);
  };
  auto put = [&](short* d, const float* v) {
    if (VEC) {
      uint4v w0, w1;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float u = v[2 * j % V], w = v[(2 * j + 1) % V];
        w0[j] = pack_bf16x2(u, w);
        w1[j] = pack_bf16x2(u - __uint_as_float(w0[j] << 16),
                            w - __uint_as_float(w0[j] & 0xffff0000u));
      }
      *(uint4v*)d = w0;
      *(uint4v*)(d + plane) = w1;
    } else {
      d[0] = f2bits(v[0]);
      d[plane] = f2bits(v[0] - bits2f(d[0]));
    }
  };
  for (int it = threadIdx.x; it < 2 * a.H * items; it += 256) {
    const int h = it / items % a.H, i = it % items * V;
    const bool key = it >= a.H * items;
    const short* src = (key ? (const short*)a.k + row * a.kst
                            : (const short*)a.q + row * a.qst) + (long)h * D;
    short* dst = (key ? x.KA : x.QA) + row * HD + (long)h * D;
    float u[V], w[V];
    get(src + half + i, w);
    if (i < half) {
      get(src + i, u);
#pragma unroll
      for (int j = 0; j < V; ++j) {
        const float c = cs[i + j], s = cs[half + i + j], y = u[j];
        u[j] = y * c - w[j] * s;
        w[j] = w[j] * c + y * s;
      }
      put(dst + i, u);
    }
    put(dst + half + i, w);
  }
}

// ---- states: U of a chunk, 64 columns per workgroup ------------------------
template <int DP, int GATE>
__global__ void __launch_bounds__(256)
memory_states_kernel(ChunkArgs x) {
  constexpr int KZ = qk_planes(GATE);
  constexpr int CPR = DP / 8, PAIRS = 32 * CPR / 256;
  constexpr int MT = DP / 32, NT = DP / 64;   // m tiles; tiles of a wave
  const MemoryArgs& a = x.a;
  const int D = a.D, E = a.E;
  const int nt = (E + 63) / 64;
  const int et = blockIdx.x % nt, h = blockIdx.x / nt % a.H;
  const int ch = blockIdx.x / nt / a.H;
  const int row0 = x.chunks[4 * ch + 1], nrow = x.chunks[4 * ch + 2];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int col = lane & 31, hi = lane >> 5;
  const int e0 = et * 64;
  const long ci = (long)ch * a.H + h;
  __shared__ __attribute__((aligned(16))) short kt[KZ][DP * 64];
  __shared__ __attribute__((aligned(16))) short vw[3][64 * 64];
  __shared__ __attribute__((aligned(16))) short vu[64 * 64];  // V^T as it is
  __shared__ float s_w[MC_L];
  {
    float w = 0.f;
    if (tid < nrow) {
      if (!fixed_decay(GATE)) {
        const long o = (long)h * x.T + row0 + tid;
        float d = x.tot[ci * 4 + wid] - x.b[o];
        for (int j = wid + 1; j < 4; ++j) d += x.tot[ci * 4 + j];
        w = GATE == TIMED ? expf(d) * x.i[o]
                          : expf(d + (x.i[o] - x.cend[ci]));
      } else {
        w = __builtin_amdgcn_exp2f((nrow - 1 - tid) * a.log2_decay[h]);
        if (GATE == TURNED) w *= a.kscale;
      }
    }
    s_w[tid] = w;
  }
  const int hk = GATE == TIMED ? h / (a.H / a.G) : h;
  const short* kp = (GATE == TURNED ? x.KA : (const short*)a.k) + (long)hk * D;
  const long kst = GATE == TURNED ? (long)a.H * D : a.kst;
  const short* vp = (const short*)a.v + (long)h * E + e0;
  const uint4v zero = {0, 0, 0, 0};
  uint4v kreg[KZ][2 * PAIRS], vreg[2];
  const int v_r = tid >> 3 << 1, v_c = (tid & 7) * 8;
  const TileWrite vtw(v_c, v_r);
  const TileRead tr(col, 0);
  auto issue = [&](int c0) {
#pragma unroll
    for (int p = 0; p < PAIRS; ++p) {
      const int it = p * 256 + tid;
      const int r = it / CPR * 2, c = it % CPR * 8;
#pragma unroll
      for (int y = 0; y < 2; ++y)
#pragma unroll
        for (int z = 0; z < KZ; ++z)
          kreg[z][2 * p + y] = c0 + r + y < nrow && c < D
              ? *(const uint4v*)(kp + ((long)z * x.T + row0 + c0 + r + y) * kst + c)
              : zero;
    }
#pragma unroll
    for (int y = 0; y < 2; ++y)
      vreg[y] = c0 + v_r + y < nrow && e0 + v_c < E
          ? *(const uint4v*)(vp + (long)(row0 + c0 + v_r + y) * a.vst + v_c)
          : zero;
  };
  f32x16 acc[NT] = {};
  float nacc = 0.f;
  const bool with_n = GATE == GATED && et == 0;
  issue(0);
  for (int c0 = 0; c0 < nrow; c0 += 64) {
    __syncthreads();
#pragma unroll
    for (int p = 0; p < PAIRS; ++p) {
      const int it = p * 256 + tid;
      const int r = it / CPR * 2, c = it % CPR * 8;
      union { uint4v u; unsigned short s[8]; } y0, y1;
      const TileWrite tw(c, r);
#pragma unroll
      for (int z = 1; z < KZ; ++z) {
        y0.u = kreg[z][2 * p];
        y1.u = kreg[z][2 * p + 1];
#pragma unroll
        for (int j = 0; j < 8; ++j)
          *(uint*)(&kt[z][tw.at(j)]) = (uint)y0.s[j] | ((uint)y1.s[j] << 16);
      }
      y0.u = silu8<GATE == DECAY>(kreg[0][2 * p]);
      y1.u = silu8<GATE == DECAY>(kreg[0][2 * p + 1]);
      if (GATE == DECAY && et == 0 && c < D) {
        short* ka = x.KA + ((long)(row0 + c0 + r) * a.H + h) * D + c;
        if (c0 + r < nrow) *(uint4v*)ka = y0.u;
        if (c0 + r + 1 < nrow) *(uint4v*)(ka + (long)a.H * D) = y1.u;
      }
#pragma unroll
      for (int j = 0; j < 8; ++j)
        *(uint*)(&kt[0][tw.at(j)]) = (uint)y0.s[j] | ((uint)y1.s[j] << 16);
    }
    {
      float f0[8], f1[8];
      unpack8(silu8<GATE == DECAY>(vreg[0]), f0);
      unpack8(silu8<GATE == DECAY>(vreg[1]), f1);
      const float w0 = s_w[c0 + v_r], w1 = s_w[c0 + v_r + 1];
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        uint w[3];
        split3(f0[j] * w0, f1[j] * w1, w);
        const int o = vtw.at(j);
        *(uint*)(vu + o) = pack_bf16x2(f0[j], f1[j]);
#pragma unroll
        for (int z = 0; z < 3; ++z) *(uint*)(&vw[z][o]) = w[z];
      }
    }
    __syncthreads();
    if (c0 + 64 < nrow) issue(c0 + 64);
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int e = (i * 256 + tid) >> 3, sl = tid & 7;
      if (e0 + e < E)
        *(uint4v*)(x.VT + (ci * E + e0 + e) * MC_L + c0 + 8 * sl) =
            *(const uint4v*)(vu + tslot(e, 8 * sl));
    }
#pragma unroll
    for (int kk = 0; kk < 4; ++kk) {
#pragma unroll
      for (int y = 0; y < NT; ++y) {
        const int tile = wid + 4 * y;
        const int m = tile % MT, n = tile / MT;
        frag_u kf[KZ];
#pragma unroll
        for (int z = 0; z < KZ; ++z)
          kf[z].u4 = *(const uint4v*)(&kt[z][tr.at(m, 2 * kk + hi)]);
#pragma unroll
        for (int z = 0; z < 3; ++z) {
          frag_u vf;
          vf.u4 = *(const uint4v*)(&vw[z][tr.at(n, 2 * kk + hi)]);
#pragma unroll
          for (int w = 0; w < KZ && w + z < 3; ++w)
            acc[y] = mfma_bf16(kf[w].bf, vf.bf, acc[y]);
        }
      }
    }
    if (with_n && tid < DP) {
#pragma unroll
      for (int s = 0; s < 64; s += 8) {
        float kv[8];
        unpack8(*(const uint4v*)(&kt[0][tslot(tid, s)]), kv);
#pragma unroll
        for (int j = 0; j < 8; ++j) nacc += s_w[c0 + s + j] * kv[j];
      }
    }
  }
  float* U = x.U + ci * E * D;
#pragma unroll
  for (int y = 0; y < NT; ++y) {
    const int tile = wid + 4 * y;
    const int m = tile % MT, e = e0 + 32 * (tile / MT) + col;
    if (e >= E) continue;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 32 * m + 8 * r + 4 * hi;
      if (d < D)
        *(f32x4*)(U + (long)e * D + d) =
            f32x4{acc[y][4 * r], acc[y][4 * r + 1], acc[y][4 * r + 2],
                  acc[y][4 * r + 3]};
    }
  }
  if (with_n && tid < D) x.N[ci * D + tid] = nacc;
}

// ---- scan over the chunks of a segment: tiles of 64 keys x 16 columns ------
template <int GATE>
__global__ void __launch_bounds__(256)
memory_scan_kernel(ChunkArgs x) {
  const MemoryArgs& a = x.a;
  const int D = a.D, E = a.E;
  const int nd = (D + 63) / 64, ne = (E + 15) / 16;
  const int dt = blockIdx.x % nd, et = blockIdx.x / nd % ne;
  const int h = blockIdx.x / nd / ne % a.H;
  const int sg = blockIdx.x / nd / ne / a.H;
  const long slot = a.seg[4 * sg];
  const int ctx = a.seg[4 * sg + 3];
  const int tid = threadIdx.x;
  const int d = dt * 64 + (tid & 15) * 4, e = et * 16 + (tid >> 4);
  const bool live = d < D && e < E;
  const int nt = (E + 31) / 32;
  float* Sp = a.S + (slot * a.H + h) * D * E;
  __shared__ float tr[64][17];
  f32x4 S = {0.f, 0.f, 0.f, 0.f};
  float m = 0.f;
  if (ctx > 0) {
    for (int i = tid; i < 64 * 16; i += 256) {
      const int dd = dt * 64 + i / 16, ee = et * 16 + i % 16;
      tr[i / 16][i % 16] = dd < D && ee < E ? Sp[(long)dd * E + ee] : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int j = 0; j < 4; ++j) S[j] = tr[(tid & 15) * 4 + j][tid >> 4];
    __syncthreads();
    if (GATE == GATED) m = a.m[(slot * a.H + h) * nt];
  }
  // the first column tile also carries n
  const bool with_n = GATE == GATED && et == 0 && tid < 64 && dt * 64 + tid < D;
  float n = 0.f;
  const long nat = (slot * a.H + h) * nt * D + dt * 64 + tid;
  if (with_n && ctx > 0) n = a.n[nat];
  // the state factors of up to 64 chunks at a time, then the chunks with the
  // next four U in flight
  constexpr int PF = 4;
  __shared__ float s_b[64], s_c[64];
  const int c0 = x.first[sg], c1 = x.first[sg + 1];
  const float l2d = fixed_decay(GATE) ? a.log2_decay[h] : 0.f;
  const long at = (long)e * D + d, step = (long)a.H * E * D;
  const float* Up = x.U + ((long)c0 * a.H + h) * E * D + at;
  f32x4 Un[PF] = {};
#pragma unroll
  for (int j = 0; j < PF; ++j)
    if (live && c0 + j < c1) Un[j] = *(const f32x4*)(Up + j * step);
  for (int cb = c0; cb < c1; cb += 64) {
    __syncthreads();
    if (tid < 64 && cb + tid < c1) {
      const long ci = (long)(cb + tid) * a.H + h;
      if (!fixed_decay(GATE)) {
        const float* tt = x.tot + ci * 4;
        const float b = tt[0] + tt[1] + tt[2] + tt[3];
        s_b[tid] = GATE == TIMED ? expf(b) : b;
        if (GATE == GATED) s_c[tid] = x.cend[ci];
      } else {
        s_b[tid] = __builtin_amdgcn_exp2f(x.chunks[4 * (cb + tid) + 2] * l2d);
      }
    }
    __syncthreads();
    const int ce = min(c1, cb + 64);
    for (int ch0 = cb; ch0 < ce; ch0 += PF) {
#pragma unroll
      for (int j = 0; j < PF; ++j) {
        const int ch = ch0 + j;
        if (ch >= ce) break;
        const long ci = (long)ch * a.H + h;
        const f32x4 U = Un[j];
        if (live && ch + PF < c1)
          Un[j] = *(const f32x4*)(Up + (long)(ch - c0 + PF) * step);
        if (live && (ch > c0 || ctx > 0)) {
          uint w0[3], w1[3];
          split3(S[0], S[1], w0);
          split3(S[2], S[3], w1);
#pragma unroll
          for (int z = 0; z < 3; ++z)
            *(uint2*)(x.P + (ci * 3 + z) * E * D + at) = uint2{w0[z], w1[z]};
        }
        float fs, us = 1.f;
        if (GATE == GATED) {
          const float bm = s_b[ch - cb] + m;
          const float mn = fmaxf(bm, s_c[ch - cb]);
          fs = expf(bm - mn);
          us = expf(s_c[ch - cb] - mn);
          if (dt == 0 && et == 0 && tid == 0) x.mst[ci] = m;
          if (with_n) {
            const long o = ci * D + dt * 64 + tid;
            const float N = x.N[o];
            x.N[o] = n;
            n = fs * n + us * N;
          }
          m = mn;
        } else {
          fs = s_b[ch - cb];
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) S[i] = fs * S[i] + us * U[i];
      }
    }
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) tr[(tid & 15) * 4 + j][tid >> 4] = S[j];
  __syncthreads();
  for (int i = tid; i < 64 * 16; i += 256) {
    const int dd = dt * 64 + i / 16, ee = et * 16 + i % 16;
    if (dd < D && ee < E) Sp[(long)dd * E + ee] = tr[i / 16][i % 16];
  }
  if (with_n)
    for (int j = 0; j < nt; ++j) a.n[nat + (long)j * D] = n;
}

// ---- outputs: 128 queries x VT columns per workgroup -----------------------
template <int DP, int VT, int GATE>
__global__ void __launch_bounds__(
    256, DP <= 128 || (VT <= 64 && GATE != TURNED) ? 2 : 1)
memory_outputs_kernel(ChunkArgs x) {
  constexpr int KZ = qk_planes(GATE);
  constexpr int NC = DP / 16, NB = VT / 32;
  constexpr int KP = DP * 2;             // K row pitch (bytes)
  constexpr int CPR = DP / 8, PAIRS = 32 * CPR / 256;
  constexpr int VN = VT / 32;            // 16-byte pieces of V^T a thread
  constexpr int KV_B = KZ * 64 * KP + VT * 64 * 2;
  constexpr int ST_B = 3 * 32 * KP;
  const MemoryArgs& a = x.a;
  const int D = a.D, E = a.E;
  const int nt = (E + VT - 1) / VT;
  const int et = blockIdx.x % nt, half = blockIdx.x / nt % 2;
  const int h = blockIdx.x / nt / 2 % a.H, ch = blockIdx.x / nt / 2 / a.H;
  const int row0 = x.chunks[4 * ch + 1], nrow = x.chunks[4 * ch + 2];
  const bool carried = x.chunks[4 * ch + 3];
  if (GATE == GATED && et == 0 && half == 0) {
    // m after the portion: nothing reads the slot's m any more
    const int sg = x.chunks[4 * ch];
    if (ch == x.first[sg + 1] - 1) {
      const long ci = (long)ch * a.H + h;
      const float* tt = x.tot + ci * 4;
      const float m = fmaxf(tt[0] + tt[1] + tt[2] + tt[3] + x.mst[ci],
                            x.cend[ci]);
      const int mt = (E + 31) / 32;
      for (int j = threadIdx.x; j < mt; j += 256)
        a.m[((long)a.seg[4 * sg] * a.H + h) * mt + j] = m;
    }
  }
  if (half * 128 >= nrow) return;        // the whole workgroup
  const int tid = threadIdx.x, lane = tid & 63;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int col = lane & 31, hi = lane >> 5;
  const int e0 = et * VT;
  const long ci = (long)ch * a.H + h;
  const int t = half * 128 + wid * 32 + col;   // place in the chunk
  const int jt = half * 2 + (wid >> 1);        // its 64-token group
  __shared__ __attribute__((aligned(16))) char
      buf[KV_B > ST_B ? KV_B : ST_B];
  char* kb = buf;
  short* vb = (short*)(buf + KZ * 64 * KP);
  __shared__ float s_col[64], s_step[GATE == TIMED ? 64 : 1];
  __shared__ float s_n[GATE == GATED ? DP : 1];
  auto kswz = [](int row, int byte) {
    return CPR >= 16 ? swz16(row, byte) : swz(row, byte);
  };

  const int hk = GATE == TIMED ? h / (a.H / a.G) : h;
  frag_u qf[KZ][NC];
#pragma unroll
  for (int z = 0; z < KZ; ++z) {
    const long r = row0 + min(t, nrow - 1);
    const short* src =
        GATE == TURNED ? x.QA + (((long)z * x.T + r) * a.H + h) * D
                       : (const short*)a.q + r * a.qst + (long)hk * D;
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      const int d = c * 16 + hi * 8;
      qf[z][c].u4 = d < D ? silu8<GATE == DECAY>(*(const uint4v*)(src + d))
                          : uint4v{0, 0, 0, 0};
    }
  }
  // row terms of the weights
  float row = 0.f, inter, em = 0.f, l2d = 0.f;
  const float qs = GATE == GATED ? a.qscale : 1.f;
  float tot[4];
  if (!fixed_decay(GATE)) {
    const long o = (long)h * x.T + row0 + min(t, nrow - 1);
    float before = GATE == GATED ? x.mst[ci] : 0.f;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      tot[j] = x.tot[ci * 4 + j];
      if (j < jt) before += tot[j];
    }
    const float bt = x.b[o];
    const float mt = GATE == GATED ? fmaxf(bt + before, x.c[o]) : 0.f;
    inter = __expf(bt + before - mt) * qs;
    row = bt - mt;
    if (GATE == GATED) em = expf(-mt);
  } else {
    l2d = a.log2_decay[h];
    inter = __builtin_amdgcn_exp2f((t + 1) * l2d);
  }

  f32x16 ot[NB] = {};
  float den = 0.f;
  if (carried) {
    // the carried state: its planes pass through LDS 32 columns at a time
    if (GATE == GATED) {
      for (int d = tid; d < DP; d += 256)
        s_n[d] = d < D ? x.N[ci * D + d] : 0.f;
    }
    const short* P = x.P + ci * 3 * E * D;
    constexpr int NP = 3 * 32 * CPR / 256;
    uint4v preg[NP];
    auto fetch = [&](int nb) {
#pragma unroll
      for (int i = 0; i < NP; ++i) {
        const int it = i * 256 + tid;
        const int c = it % CPR * 8, r = it / CPR;     // r: plane * 32 + row
        const int e = e0 + 32 * nb + (r & 31);
        preg[i] = e < E && c < D
            ? *(const uint4v*)(P + ((long)(r >> 5) * E + e) * D + c)
            : uint4v{0, 0, 0, 0};
      }
    };
    fetch(0);
#pragma unroll
    for (int nb = 0; nb < NB; ++nb) {
      if (e0 + 32 * nb >= E) continue;   // uniform
      __syncthreads();
#pragma unroll
      for (int i = 0; i < NP; ++i) {
        const int it = i * 256 + tid;
        const int c = it % CPR * 8, r = it / CPR;
        *(uint4v*)(buf + r * KP + kswz(r & 31, c * 2)) = preg[i];
      }
      __syncthreads();
      if (nb + 1 < NB) fetch(nb + 1);
#pragma unroll
      for (int z = 0; z < 3; ++z)
#pragma unroll
        for (int c = 0; c < NC; ++c) {
          frag_u sf;
          sf.u4 = *(const uint4v*)(buf + (z * 32 + col) * KP +
                                   kswz(col, (c * 16 + hi * 8) * 2));
#pragma unroll
          for (int w = 0; w < KZ && w + z < 3; ++w)
            ot[nb] = mfma_bf16(sf.bf, qf[w][c].bf, ot[nb]);
        }
      ot[nb] *= inter;
    }
    if (GATE == GATED) {
#pragma unroll
      for (int c = 0; c < NC; ++c) {
        float qv[8];
        unpack8(qf[0][c].u4, qv);
#pragma unroll
        for (int j = 0; j < 8; ++j) den += qv[j] * s_n[c * 16 + hi * 8 + j];
      }
      den *= inter;
    }
  }

  // ---- keys of the chunk, 64 at a time, from the newest back ---------------
  const short* kp =
      (fixed_decay(GATE) ? x.KA : (const short*)a.k) + (long)hk * D;
  const long kst = fixed_decay(GATE) ? (long)a.H * D : a.kst;
  const short* vp = x.VT + (ci * E + e0) * MC_L;
  const uint4v zero = {0, 0, 0, 0};
  uint4v kreg[KZ][2 * PAIRS], vreg[VN];
  float colr = 0.f, stepr = 0.f;
  auto issue = [&](int J) {
    const int c0 = 64 * J;
#pragma unroll
    for (int p = 0; p < 2 * PAIRS; ++p) {
      const int it = p * 256 + tid;
      const int r = it / CPR, c = it % CPR * 8;
#pragma unroll
      for (int z = 0; z < KZ; ++z)
        kreg[z][p] = c0 + r < nrow && c < D
            ? *(const uint4v*)(kp + ((long)z * x.T + row0 + c0 + r) * kst + c)
            : zero;
    }
#pragma unroll
    for (int p = 0; p < VN; ++p) {
      const int e = (p * 256 + tid) >> 3;
      vreg[p] = e0 + e < E
          ? *(const uint4v*)(vp + (long)e * MC_L + c0 + 8 * (tid & 7)) : zero;
    }
    if (!fixed_decay(GATE) && tid < 64) {
      colr = -INFINITY;
      stepr = 0.f;
      if (c0 + tid < nrow) {
        const long o = (long)h * x.T + row0 + c0 + tid;
        stepr = x.i[o];
        colr = GATE == TIMED ? -x.b[o] : stepr - x.b[o];
      }
    }
  };
  const TileRead vr(col, 4 * hi);
  const int J1 = min(half * 2 + 1, (nrow - 1) / 64);
  issue(J1);
  for (int J = J1; J >= 0; --J) {
    __syncthreads();
#pragma unroll
    for (int p = 0; p < 2 * PAIRS; ++p) {
      const int it = p * 256 + tid;
      const int r = it / CPR, c = it % CPR * 8;
#pragma unroll
      for (int z = 0; z < KZ; ++z)
        *(uint4v*)(kb + (z * 64 + r) * KP + kswz(r, c * 2)) = kreg[z][p];
    }
#pragma unroll
    for (int p = 0; p < VN; ++p)
      *(uint4v*)(vb + tslot((p * 256 + tid) >> 3, 8 * (tid & 7))) = vreg[p];
    if (!fixed_decay(GATE) && tid < 64) s_col[tid] = colr;
    if (GATE == TIMED && tid < 64) s_step[tid] = stepr;
    __syncthreads();
    if (J > 0) issue(J - 1);
    if (J > jt || half * 128 + wid * 32 >= nrow) continue;  // wave-uniform

    // row part of the exponent for keys of group J
    float base = row;
    if (!fixed_decay(GATE) && J < jt) {
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (j >= J && j < jt) base += tot[j];
    }
    // 32 keys at a time keeps the registers for two workgroups per CU
#pragma unroll 1
    for (int k2 = 0; k2 < 2; ++k2) {
      const int kr = col + 32 * k2;
      f32x16 acc = {};
#pragma unroll
      for (int c = 0; c < NC; ++c) {
#pragma unroll
        for (int z = 0; z < KZ; ++z) {
          frag_u kf;
          kf.u4 = *(const uint4v*)(kb + (z * 64 + kr) * KP +
                                   kswz(kr, (c * 16 + hi * 8) * 2));
#pragma unroll
          for (int w = 0; w < KZ && w + z < 2; ++w)
            acc = mfma_bf16(kf.bf, qf[w][c].bf, acc);
        }
      }
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int s = 32 * k2 + acc_row(r, hi);
        float w;
        if (GATE == TIMED) w = __expf(base + s_col[s]) * s_step[s];
        else if (GATE == GATED) w = __expf(base + s_col[s]) * qs;
        else w = __builtin_amdgcn_exp2f((float)(t - 64 * J - s) * l2d);
        if (GATE == TURNED) w *= a.kscale;
        if (J == jt && 64 * J + s > t) w = 0.f;
        acc[r] *= w;
        if (GATE == GATED) den += acc[r];
      }
#pragma unroll
      for (int cc = 0; cc < 2; ++cc) {
        frag_u pf[3];
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          uint w[3];
          split3(acc[8 * cc + 2 * u], acc[8 * cc + 2 * u + 1], w);
#pragma unroll
          for (int z = 0; z < 3; ++z) pf[z].u[u] = w[z];
        }
        const int slot = 4 * k2 + 2 * cc;
#pragma unroll
        for (int nb = 0; nb < NB; ++nb) {
          frag_u vf;
          *(uint2*)&vf.u[0] = *(const uint2*)(vb + vr.at(nb, slot));
          *(uint2*)&vf.u[2] = *(const uint2*)(vb + vr.at(nb, slot + 1));
#pragma unroll
          for (int z = 0; z < 3; ++z)
            ot[nb] = mfma_bf16(vf.bf, pf[z].bf, ot[nb]);
        }
      }
    }
  }

  float inv = 1.f;
  if (GATE == GATED) {
    den += __shfl_xor(den, 32, 64);
    inv = 1.f / (fmaxf(fabsf(den), em) + GATED_EPS);
  }
  if (GATE == TURNED && a.z) {           // the head's norm; e0 is 0
    float sq = 0.f;
#pragma unroll
    for (int nb = 0; nb < NB; ++nb)
#pragma unroll
      for (int r = 0; r < 16; ++r) sq += ot[nb][r] * ot[nb][r];
    sq += __shfl_xor(sq, 32, 64);
    inv = 1.f / sqrtf(sq / E + x.norm_eps);
  }
  if (t >= nrow) return;
  const float skip = GATE == TIMED ? bits2f(((const short*)a.skip)[h]) : 0.f;
  short* dst = (short*)a.out + ((long)(row0 + t) * a.H + h) * E + e0;
#pragma unroll
  for (int nb = 0; nb < NB; ++nb)
#pragma unroll
    for (int rg = 0; rg < 4; ++rg) {
      const int e = 32 * nb + 8 * rg + 4 * hi;
      if (e0 + e >= E) continue;
      float o[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) o[j] = ot[nb][4 * rg + j] * inv;
      if (GATE == TURNED && a.z) {
        float z[4];
        load4((const short*)a.z + (long)(row0 + t) * a.zst + (long)h * E + e, z);
#pragma unroll
        for (int j = 0; j < 4; ++j) o[j] *= silu_f(z[j]);
      }
      if (GATE == TIMED) {
        float v[4], z[4];
        const long at = (long)h * E + e0 + e;
        load4((const short*)a.v + (long)(row0 + t) * a.vst + at, v);
        load4((const short*)a.z + (long)(row0 + t) * a.zst + at, z);
#pragma unroll
        for (int j = 0; j < 4; ++j) o[j] = (o[j] + skip * v[j]) * silu_f(z[j]);
      }
      *(uint2*)(dst + e) = uint2{pack_bf16x2(o[0], o[1]),
                                 pack_bf16x2(o[2], o[3])};
    }
}

// wider column tiles read the keys less often, as long as the accumulators
// leave registers for two workgroups per CU
template <int DP, int GATE>
static void launch_chunks(const ChunkArgs& x, hipStream_t stream) {
  const MemoryArgs& a = x.a;
  const long ch = (long)x.n_chunks * a.H;
  if (!fixed_decay(GATE)) memory_gates_kernel<GATE><<<ch, MC_L, 0, stream>>>(x);
  if (GATE == TURNED) {
    const size_t lds = a.rot * sizeof(float);
    const long rows = (long)x.n_chunks * MC_L;
    if (a.rot % 16 == 0) memory_turn_kernel<true><<<rows, 256, lds, stream>>>(x);
    else memory_turn_kernel<false><<<rows, 256, lds, stream>>>(x);
  }
  memory_states_kernel<DP, GATE>
      <<<ch * ((a.E + 63) / 64), 256, 0, stream>>>(x);
  memory_scan_kernel<GATE><<<(long)x.n_seg * a.H * ((a.D + 63) / 64) *
                                 ((a.E + 15) / 16), 256, 0, stream>>>(x);
  if (a.E <= 64 || DP > 128)
    memory_outputs_kernel<DP, 64, GATE>
        <<<ch * 2 * ((a.E + 63) / 64), 256, 0, stream>>>(x);
  else
    memory_outputs_kernel<DP, (DP > 128 ? 64 : 128), GATE>
        <<<ch * 2 * ((a.E + 127) / 128), 256, 0, stream>>>(x);
}

// bf16; D and E multiples of 8 with D <= 256; 16-byte aligned rows
extern "C" int sv_memory_chunks(const ChunkArgs* x, int gating,
                                hipStream_t stream) {
  if (x->n_seg <= 0) return 0;
  if (gating == TURNED &&
      (x->a.rot % 2 || x->a.rot > x->a.D ||
       (x->a.z && (x->a.E > 128 || (x->a.E > 64 && x->a.D > 128)))))
    return 1;
#define MC(P)                                                     \
  do {                                                            \
    if (gating == GATED) launch_chunks<P, GATED>(*x, stream);     \
    else if (gating == TIMED) launch_chunks<P, TIMED>(*x, stream); \
    else if (gating == TURNED) launch_chunks<P, TURNED>(*x, stream); \
    else launch_chunks<P, DECAY>(*x, stream);                     \
  } while (0)
  if (x->a.D <= 64) MC(64);
  else if (x->a.D <= 128) MC(128);
  else if (x->a.D <= 256) MC(256);
  else return 1;
#undef MC
  return (int)hipGetLastError();
}
