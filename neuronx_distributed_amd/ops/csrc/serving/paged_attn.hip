// Attention over a paged KV cache for ragged batches.
//
// Cache layout: K [page][kv head][64][D], V [page][kv head][64][E]; a
// request's block table maps position / 64 to a page.  Visibility of key j
// for the query at position i:  j <= i and (i - j < window or j < keep).
// window <= 0 means plain causal.  Sizes D and E need not be equal.
//
// Scores and the softmax may be modified (ScoreArgs): a factor a head, a soft
// cap, a bias that falls with the distance, a sink in the denominator; the
// output may pass through one gate a head.
//
//   sv_kv_append   writes the K/V rows of a step into their pages
//   sv_qkv_append  the same with rotation and norm of queries and keys and with
//                  values mixed with another layer's
//   sv_attn_rows   one query row per workgroup group: single-token decoding
//                  (the row's own K/V is appended here) and the 32-bit mode
//   sv_attn_tiles  MFMA flash kernel over 128-row tiles for prompt portions

#include "serving.h"

#define NEG_BIG (-1e30f)

// ---------------------------------------------------------------------------
// append
// ---------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256)
kv_append_kernel(const T* __restrict__ k, const T* __restrict__ v, long kst,
                 long vst, T* __restrict__ kc, T* __restrict__ vc,
                 const int* __restrict__ pos, const int* __restrict__ seq,
                 const int* __restrict__ bt, int MB, int G, int D, int E) {
  const int t = blockIdx.x;
  const int p = pos[t];
  const long page = bt[(long)seq[t] * MB + p / SV_PAGE];
  const int in_page = p % SV_PAGE;
  for (int i = threadIdx.x; i < G * D; i += 256)
    kc[((page * G + i / D) * SV_PAGE + in_page) * D + i % D] = k[t * kst + i];
  for (int i = threadIdx.x; i < G * E; i += 256)
    vc[((page * G + i / E) * SV_PAGE + in_page) * E + i % E] = v[t * vst + i];
}

// 8 elements a thread when every row is a multiple of 8 elements
template <typename T>
__global__ void __launch_bounds__(256)
kv_append_vec_kernel(const T* __restrict__ k, const T* __restrict__ v,
                     long kst, long vst, T* __restrict__ kc,
                     T* __restrict__ vc, const int* __restrict__ pos,
                     const int* __restrict__ seq, const int* __restrict__ bt,
                     int MB, int G, int D, int E) {
  const int t = blockIdx.x;
  const int p = pos[t];
  const long page = bt[(long)seq[t] * MB + p / SV_PAGE];
  const int in_page = p % SV_PAGE;
  constexpr int NW = 8 * sizeof(T) / 16;
  for (int i = threadIdx.x * 8; i < G * D; i += 256 * 8) {
    const uint4v* s = (const uint4v*)(k + t * kst + i);
    uint4v* d = (uint4v*)(kc + ((page * G + i / D) * SV_PAGE + in_page) * D +
                          i % D);
#pragma unroll
    for (int j = 0; j < NW; ++j) d[j] = s[j];
  }
  for (int i = threadIdx.x * 8; i < G * E; i += 256 * 8) {
    const uint4v* s = (const uint4v*)(v + t * vst + i);
    uint4v* d = (uint4v*)(vc + ((page * G + i / E) * SV_PAGE + in_page) * E +
                          i % E);
#pragma unroll
    for (int j = 0; j < NW; ++j) d[j] = s[j];
  }
}

extern "C" int sv_kv_append(const void* k, const void* v, long kst, long vst,
                            void* kc, void* vc, const int* pos,
                            const int* seq, const int* bt, int MB, int T,
                            int G, int D, int E, int vec, int f32,
                            hipStream_t stream) {
  if (T <= 0) return 0;
#define KA(K, TT)                                                            \
  K<TT><<<T, 256, 0, stream>>>((const TT*)k, (const TT*)v, kst, vst,         \
                               (TT*)kc, (TT*)vc, pos, seq, bt, MB, G, D, E)
  if (f32) { if (vec) KA(kv_append_vec_kernel, float); else KA(kv_append_kernel, float); }
  else     { if (vec) KA(kv_append_vec_kernel, short); else KA(kv_append_kernel, short); }
#undef KA
  return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// append with what comes before the attention.  LPH lanes own a head of a row
// (8 elements each).  Queries are changed in place, keys and values go into
// their pages only.
// ---------------------------------------------------------------------------
struct QkvArgs {
  void* q;
  const void *k, *v;
  long qst, kst, vst;
  const double* freq;       // [rot / 2] radians a position: elements 2i and
                            //   2i + 1 turn; or null
  const void *qw, *kw;      // [D] weights of the norm, or null
  const void* first;        // values to mix in, or null
  long fst;
  const void* mix;          // their share (one number)
  void *kc, *vc;
  const int *pos, *seq, *bt;
  int MB, T, H, G, D, E, rot;
  int norm;                 // queries and keys over their root mean square
  int temp_every;           // > 0: queries times 1 + coef ln(floor((p + 1) /
  float temp_coef, eps;     //   every) + 1)
};

template <typename T, int LPH, bool VEC>
__global__ void __launch_bounds__(256) qkv_append_kernel(QkvArgs a) {
  constexpr int PER = 256 / LPH;         // heads of a workgroup
  const int heads = a.H + 2 * a.G;
  const long item = (long)blockIdx.x * PER + threadIdx.x / LPH;
  const long row = min(item / heads, (long)a.T - 1);
  const bool live = item < (long)a.T * heads;
  const int hh = item % heads, d0 = threadIdx.x % LPH * 8;
  const int p = a.pos[row];
  const long page = a.bt[(long)a.seq[row] * a.MB + p / SV_PAGE];
  const bool is_q = hh < a.H, is_v = hh >= a.H + a.G;
  const int g = is_q ? 0 : is_v ? hh - a.H - a.G : hh - a.H;
  const int size = is_v ? a.E : a.D;
  const int n = min(8, size - d0);       // elements of this lane; <= 0: none
  const T* src = is_q   ? (const T*)a.q + row * a.qst + (long)hh * a.D
                 : is_v ? (const T*)a.v + row * a.vst + (long)g * a.E
                        : (const T*)a.k + row * a.kst + (long)g * a.D;
  float x[8];
  load8<VEC>(src + d0, n, x);
  if (is_v && a.first) {
    const float m = to_f(((const T*)a.mix)[0]);
    float f[8];
    load8<VEC>((const T*)a.first + row * a.fst + (long)g * a.E + d0, n, f);
#pragma unroll
    for (int j = 0; j < 8; ++j) x[j] = (1.f - m) * x[j] + m * f[j];
  }
  if (!is_v && a.freq) {
#pragma unroll
    for (int j = 0; j < 8; j += 2) {
      if (d0 + j >= a.rot) continue;
      float c, s;
      turn(a.freq[(d0 + j) / 2], p, &c, &s);
      const float u = x[j], w = x[j + 1];
      x[j] = u * c - w * s;
      x[j + 1] = w * c + u * s;
    }
  }
  if (a.norm) {                          // all lanes: values join the shuffles
    float sq = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) sq += x[j] * x[j];
#pragma unroll
    for (int off = LPH / 2; off > 0; off >>= 1) sq += __shfl_xor(sq, off, 64);
    if (!is_v) {
      const float rstd = 1.f / sqrtf(sq / a.D + a.eps);
      const T* w = (const T*)(is_q ? a.qw : a.kw);
      float u[8];
      if (w) load8<VEC>(w + d0, n, u);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[j] *= w ? rstd * u[j] : rstd;
    }
  }
  if (is_q && a.temp_every > 0) {
    const float t = 1.f + a.temp_coef * logf((float)((p + 1) / a.temp_every + 1));
#pragma unroll
    for (int j = 0; j < 8; ++j) x[j] *= t;
  }
  if (!live || n <= 0) return;
  const long at = (page * a.G + g) * SV_PAGE + p % SV_PAGE;
  T* dst = is_q   ? (T*)a.q + row * a.qst + (long)hh * a.D
           : is_v ? (T*)a.vc + at * a.E : (T*)a.kc + at * a.D;
  if (VEC) {
    store4(dst + d0, x);
    store4(dst + d0 + 4, x + 4);
  } else {
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (j < n) from_f(dst[d0 + j], x[j]);
  }
}

// D and E at most 512; vec: D, E, strides and bases in 8 elements
extern "C" int sv_qkv_append(const QkvArgs* a, int vec, int f32,
                             hipStream_t stream) {
  if (a->T <= 0) return 0;
  if (a->rot % 2 || a->rot > a->D) return 1;
  const int big = a->D > a->E ? a->D : a->E;
  const long items = (long)a->T * (a->H + 2 * a->G);
#define QA(T, L, V)                                              \
  qkv_append_kernel<T, L, V>                                     \
      <<<(items + 256 / L - 1) / (256 / L), 256, 0, stream>>>(*a)
#define QAV(L)                                                   \
  do {                                                           \
    if (f32) { if (vec) QA(float, L, true); else QA(float, L, false); } \
    else     { if (vec) QA(short, L, true); else QA(short, L, false); } \
  } while (0)
  if (big <= 64) QAV(8);
  else if (big <= 128) QAV(16);
  else if (big <= 256) QAV(32);
  else if (big <= 512) QAV(64);
  else return 1;
#undef QAV
#undef QA
  return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// scores: s = q.k scale temp_h; s <- cap tanh(s / cap); s <- s - slope_h
// (i - j); the denominator also holds exp(sink_h); the output of head h is
// multiplied by sigmoid(gate[row][h]).  What is null or zero is left out.
// ---------------------------------------------------------------------------
struct ScoreArgs {
  const void *temp, *sink;  // [H], T
  const float* slope;       // [H]
  const void* gate;         // [rows][H], T
  long gst;
  float cap;
};

// ---------------------------------------------------------------------------
// rows
// ---------------------------------------------------------------------------
struct RowsArgs {
  const void *q, *k, *v;       // row 0 of the step's projections
  long qst, kst, vst;          // row strides (elements)
  void *kc, *vc;               // cache
  long kcs, vcs;               // elements from one cached row to the next
  const int *pos, *seq, *bt;   // per row: position, sequence; block table
  float* part;                 // [rows][H][splits][E + 2] or null (1 split)
  void* out;                   // [rows][H * E]
  int MB, rows, H, G, D, E, splits, append, window, keep;
  float scale;
  ScoreArgs mod;
};

// tanh, in the 32-bit mode to the last digits, else to 1e-7
__device__ __forceinline__ float tanh_t(float x, float) { return tanhf(x); }
__device__ __forceinline__ float tanh_t(float x, short) {
  return 1.f - 2.f * __builtin_amdgcn_rcpf(
                         1.f + __builtin_amdgcn_exp2f(2.f * SV_LOG2E * x));
}

// LPR lanes own one key row (DPL dims each); RC query heads share the row.
template <bool VEC, int DPL, typename T>
__device__ __forceinline__ void load_dims(const T* p, int n, float* v) {
#pragma unroll
  for (int j = 0; j < DPL; j += 8) load8<VEC>(p + j, n - j, v + j);
}

// MOD: scores and softmax as ScoreArgs say; without it they are plain.
template <bool MOD, typename T, int LPR, int RC, bool VEC, int DPL = 8>
__global__ void __launch_bounds__(256, RC <= 4 && DPL == 8 ? 4 : 1)
attn_rows_kernel(RowsArgs a) {
  constexpr int NR = 64 / LPR;     // key rows of one wave step
  constexpr int DV = LPR * DPL;
  const int rep = a.H / a.G;
  const int nrc = (rep + RC - 1) / RC;
  const int split = blockIdx.x % a.splits;
  const int unit = blockIdx.x / a.splits;
  const int rc = unit % nrc;
  const int g = unit / nrc % a.G;
  const int row = unit / nrc / a.G;
  const int lane = threadIdx.x & 63;
  const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int hl = lane % LPR, sub = lane / LPR;
  const int d0 = DPL * hl;
  // dims of this lane; <= 0: none
  const int nd = min(DPL, a.D - d0), ne = min(DPL, a.E - d0);
  const int D = a.D, E = a.E;

  const int i_pos = a.pos[row];
  const int* bt = a.bt + (long)a.seq[row] * a.MB;

  float qv[RC][DPL];
#pragma unroll
  for (int r = 0; r < RC; ++r) {
    const int h = g * rep + min(rc * RC + r, rep - 1);
    load_dims<VEC, DPL>((const T*)a.q + row * a.qst + (long)h * D + d0, nd, qv[r]);
  }
  // scores in units of log 2; of the cap, if there is one
  const float cap = MOD ? a.mod.cap : 0.f;
  const float s2 = cap > 0.f ? a.scale / cap : a.scale * SV_LOG2E;
  float slope[RC];
#pragma unroll
  for (int r = 0; r < RC; ++r) {
    float t = s2;
    if (MOD) {
      const int h = g * rep + min(rc * RC + r, rep - 1);
      if (a.mod.temp) t *= to_f(((const T*)a.mod.temp)[h]);
      // the same for all lanes: not in a vector register
      slope[r] = __uint_as_float(__builtin_amdgcn_readfirstlane(__float_as_uint(
          a.mod.slope ? a.mod.slope[h] * SV_LOG2E : 0.f)));
    }
#pragma unroll
    for (int j = 0; j < DPL; ++j) qv[r][j] *= t;
  }

  const T* kn = (const T*)a.k + row * a.kst + (long)g * D;
  const T* vn = (const T*)a.v + row * a.vst + (long)g * E;
  if (a.append && split == 0 && rc == 0) {
    const long page = bt[i_pos / SV_PAGE];
    const long base = (page * a.G + g) * SV_PAGE + i_pos % SV_PAGE;
    for (int i = threadIdx.x; i < D; i += 256)
      ((T*)a.kc)[base * a.kcs + i] = kn[i];
    for (int i = threadIdx.x; i < E; i += 256)
      ((T*)a.vc)[base * a.vcs + i] = vn[i];
  }

  // visible keys as one list: the kept first ones, then the window.  With
  // append, the row's own key is handled from registers at the end.
  const int lo = a.window > 0 ? max(0, i_pos - a.window + 1) : 0;
  const int nfirst = min(a.keep, lo);
  const int total = nfirst + (i_pos - lo) + (a.append ? 0 : 1);
  const int per = (total + a.splits - 1) / a.splits;
  const int k0 = split * per, k1 = min(total, k0 + per);

  float m[RC], l[RC], o[RC][DPL];
#pragma unroll
  for (int r = 0; r < RC; ++r) {
    m[r] = NEG_BIG;
    l[r] = 0.f;
#pragma unroll
    for (int j = 0; j < DPL; ++j) o[r][j] = 0.f;
  }

  auto fetch = [&](int idx, float* kf, float* vf) {
    const int j = idx < nfirst ? idx : lo + idx - nfirst;
    const long base =
        ((long)bt[j / SV_PAGE] * a.G + g) * SV_PAGE + j % SV_PAGE;
    load_dims<VEC, DPL>((const T*)a.kc + base * a.kcs + d0, nd, kf);
    load_dims<VEC, DPL>((const T*)a.vc + base * a.vcs + d0, ne, vf);
  };
  auto absorb = [&](const float* kf, const float* vf, bool live, int away) {
    float s[RC];
#pragma unroll
    for (int r = 0; r < RC; ++r) {
      s[r] = 0.f;
#pragma unroll
      for (int j = 0; j < DPL; ++j) s[r] += qv[r][j] * kf[j];
    }
#pragma unroll
    for (int off = LPR / 2; off > 0; off >>= 1)
#pragma unroll
      for (int r = 0; r < RC; ++r) s[r] += __shfl_xor(s[r], off, 64);
    if (MOD) {
      if (cap > 0.f)
#pragma unroll
        for (int r = 0; r < RC; ++r) s[r] = cap * SV_LOG2E * tanh_t(s[r], T());
#pragma unroll
      for (int r = 0; r < RC; ++r) s[r] -= slope[r] * away;
    }
#pragma unroll
    for (int r = 0; r < RC; ++r) {
      const float mn = live ? fmaxf(m[r], s[r]) : m[r];
      const float al = __builtin_amdgcn_exp2f(m[r] - mn);
      const float p = live ? __builtin_amdgcn_exp2f(s[r] - mn) : 0.f;
      m[r] = mn;
      l[r] = l[r] * al + p;
#pragma unroll
      for (int j = 0; j < DPL; ++j) o[r][j] = o[r][j] * al + p * vf[j];
    }
  };

  float kf[DPL], vf[DPL];
  int idx = k0 + wid * NR + sub;
#pragma unroll
  for (int j = 0; j < DPL; ++j) kf[j] = vf[j] = 0.f;
  if (idx < k1) fetch(idx, kf, vf);
  for (int b = k0 + wid * NR; b < k1; b += 4 * NR, idx += 4 * NR) {
    float kx[DPL], vx[DPL];
#pragma unroll
    for (int j = 0; j < DPL; ++j) kx[j] = vx[j] = 0.f;
    if (idx + 4 * NR < k1) fetch(idx + 4 * NR, kx, vx);
    absorb(kf, vf, idx < k1,
           MOD ? i_pos - (idx < nfirst ? idx : lo + idx - nfirst) : 0);
#pragma unroll
    for (int j = 0; j < DPL; ++j) {
      kf[j] = kx[j];
      vf[j] = vx[j];
    }
  }
  if (a.append && split == 0 && wid == 0) {
    load_dims<VEC, DPL>(kn + d0, nd, kf);
    load_dims<VEC, DPL>(vn + d0, ne, vf);
    absorb(kf, vf, sub == 0, 0);
  }

  // fold the NR row groups of the wave, then the 4 waves
#pragma unroll
  for (int off = 32; off >= LPR; off >>= 1)
#pragma unroll
    for (int r = 0; r < RC; ++r) {
      const float m2 = __shfl_xor(m[r], off, 64);
      const float l2 = __shfl_xor(l[r], off, 64);
      const float mn = fmaxf(m[r], m2);
      const float c1 = __builtin_amdgcn_exp2f(m[r] - mn);
      const float c2 = __builtin_amdgcn_exp2f(m2 - mn);
      m[r] = mn;
      l[r] = l[r] * c1 + l2 * c2;
#pragma unroll
      for (int j = 0; j < DPL; ++j)
        o[r][j] = o[r][j] * c1 + __shfl_xor(o[r][j], off, 64) * c2;
    }
  __shared__ float so[4][RC][DV];
  __shared__ float sml[4][RC][2];
  if (sub == 0) {
#pragma unroll
    for (int r = 0; r < RC; ++r) {
#pragma unroll
      for (int j = 0; j < DPL; ++j) so[wid][r][d0 + j] = o[r][j];
      if (hl == 0) {
        sml[wid][r][0] = m[r];
        sml[wid][r][1] = l[r];
      }
    }
  }
  __syncthreads();
  for (int it = threadIdx.x; it < RC * DV; it += 256) {
    const int r = it / DV, e = it % DV;
    if (rc * RC + r >= rep || e >= E) continue;
    float mm = NEG_BIG;
#pragma unroll
    for (int w = 0; w < 4; ++w) mm = fmaxf(mm, sml[w][r][0]);
    float ll = 0.f, oo = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float c = __builtin_amdgcn_exp2f(sml[w][r][0] - mm);
      ll += sml[w][r][1] * c;
      oo += so[w][r][e] * c;
    }
    const int h = g * rep + rc * RC + r;
    if (MOD && a.mod.sink && split == 0) {   // once for all splits
      const float sink = to_f(((const T*)a.mod.sink)[h]) * SV_LOG2E;
      const float mn = fmaxf(mm, sink);
      const float c = __builtin_amdgcn_exp2f(mm - mn);
      ll = ll * c + __builtin_amdgcn_exp2f(sink - mn);
      oo *= c;
      mm = mn;
    }
    if (MOD && a.mod.gate)
      oo *= sigmoid_f(to_f(((const T*)a.mod.gate)[row * a.mod.gst + h]));
    if (a.splits == 1) {
      from_f(((T*)a.out)[((long)row * a.H + h) * E + e], oo / ll);
    } else {
      float* p = a.part +
                 (((long)row * a.H + h) * a.splits + split) * (E + 2);
      p[e] = oo;
      if (e == 0) {
        p[E] = mm;
        p[E + 1] = ll;
      }
    }
  }
}

// One workgroup = one query row and head, 64 V columns; its four waves take
// every fourth split.  At most 64 splits.
template <typename T, int V>
__global__ void __launch_bounds__(256)
attn_rows_merge_kernel(const float* __restrict__ part, T* __restrict__ out,
                       int splits, int E) {
  __shared__ float coef[64], sum[4][64][V];
  const long rh = blockIdx.x;
  const int lane = threadIdx.x & 63;
  const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const float* p = part + rh * splits * (E + 2);
  if (wid == 0) {
    float m = NEG_BIG, l = 0.f;
    if (lane < splits) {
      m = p[(long)lane * (E + 2) + E];
      l = p[(long)lane * (E + 2) + E + 1];
    }
    float mm = m;
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) mm = fmaxf(mm, __shfl_xor(mm, off, 64));
    const float w = __builtin_amdgcn_exp2f(m - mm);
    l *= w;
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) l += __shfl_xor(l, off, 64);
    coef[lane] = w / l;
  }
  __syncthreads();
  const int e = (blockIdx.y * 64 + lane) * V;
  float acc[V] = {};
  if (e < E) {
    const float* src = p + e;
#pragma unroll 8
    for (int s = wid; s < splits; s += 4) {
      const float c = coef[s];
#pragma unroll
      for (int j = 0; j < V; ++j) acc[j] += c * src[(long)s * (E + 2) + j];
    }
  }
#pragma unroll
  for (int j = 0; j < V; ++j) sum[wid][lane][j] = acc[j];
  __syncthreads();
  if (wid > 0 || e >= E) return;
#pragma unroll
  for (int j = 0; j < V; ++j)
    from_f(out[rh * E + e + j], sum[0][lane][j] + sum[1][lane][j] +
                                    sum[2][lane][j] + sum[3][lane][j]);
}

extern "C" int sv_attn_merge(const float* part, void* out, long rows,
                             int splits, int E, int f32, hipStream_t stream) {
  if (splits > 64) return 1;
  const int v = E % 2 ? 1 : 2;
  const dim3 grid(rows, (E + 64 * v - 1) / (64 * v));
#define AM(T, V) attn_rows_merge_kernel<T, V><<<grid, 256, 0, stream>>>( \
      part, (T*)out, splits, E)
  if (f32) { if (v == 2) AM(float, 2); else AM(float, 1); }
  else     { if (v == 2) AM(short, 2); else AM(short, 1); }
#undef AM
  return (int)hipGetLastError();
}

template <bool MOD, typename T>
static int launch_rows(const RowsArgs& a, int vec, hipStream_t stream) {
  const int rep = a.H / a.G;
  const int big = a.D > a.E ? a.D : a.E;
  const int rcn = big > 512 ? (rep > 1 ? 2 : 1)
                            : rep >= 8 ? 8 : rep > 2 ? 4 : rep;
  const int nrc = (rep + rcn - 1) / rcn;
  const long grid = (long)a.rows * a.G * nrc * a.splits;
#define AR(L, ...) \
  attn_rows_kernel<MOD, T, L, __VA_ARGS__><<<grid, 256, 0, stream>>>(a)
#define ARV(L, R) do { if (vec) AR(L, R, true); else AR(L, R, false); } while (0)
#define ARR(L)                                                         \
  do {                                                                 \
    if (rcn == 8) ARV(L, 8); else if (rcn == 4) ARV(L, 4);             \
    else if (rcn == 2) ARV(L, 2); else ARV(L, 1);                      \
  } while (0)
  if (big <= 64) ARR(8);
  else if (big <= 128) ARR(16);
  else if (big <= 256) ARR(32);
  else if (big <= 512) ARR(64);
  else if (big <= 1024) {
    if (rcn == 2) { if (vec) AR(64, 2, true, 16); else AR(64, 2, false, 16); }
    else { if (vec) AR(64, 1, true, 16); else AR(64, 1, false, 16); }
  } else return 1;
#undef ARR
#undef ARV
#undef AR
  if (a.splits > 1)
    return sv_attn_merge(a.part, a.out, (long)a.rows * a.H, a.splits, a.E,
                         sizeof(T) == 4, stream);
  return (int)hipGetLastError();
}

extern "C" int sv_attn_rows(const RowsArgs* a, int vec, int f32,
                            hipStream_t stream) {
  if (a->rows <= 0) return 0;
  const ScoreArgs& m = a->mod;
  const bool mod = m.temp || m.sink || m.slope || m.gate || m.cap > 0.f;
  if (f32)
    return mod ? launch_rows<true, float>(*a, vec, stream)
               : launch_rows<false, float>(*a, vec, stream);
  return mod ? launch_rows<true, short>(*a, vec, stream)
             : launch_rows<false, short>(*a, vec, stream);
}

// ---------------------------------------------------------------------------
// tiles: bf16 MFMA flash attention for prompt portions
//
// One workgroup = 4 waves x 32 query rows of one head; a key tile is one
// cache page.  S^T = K Q^T keeps every softmax statistic lane-local (a lane
// owns one query row).  The weights stay 32-bit: P is split exactly into
// NP bf16 planes (3 planes carry the full 24-bit significand) and V enters
// once per plane.  P never leaves registers: the accumulator's row order
// {4 hi + 0..3, 8 + 4 hi + 0..3} of a 16-key chunk is used as the
// contraction order of P V, and V^T is read from LDS in the same order
// (transposing loads).
// ---------------------------------------------------------------------------
//
// A key may end in columns that all heads share (kr): the rotated part of
// latent attention, whose other columns are expanded into a workspace first.
// The output may pass through sigmoid(gate).
struct TilesArgs {
  const short* q;
  long qst;                 // row stride of q
  const short *kc, *vc, *kr;
  long kpage, khead, krow;  // elements between pages, heads, rows
  long vpage, vhead, vrow;
  long rrow;                // between rows of kr (pages follow each other)
  const short* gate;        // [T][H * E] or null
  long gst;
  const int* tiles;         // [n_tiles][4]: seq, first row, rows, position
  const int* bt;
  short* out;               // [T][H * E]
  int MB, H, G, D, E, DS;   // DS: columns of a key before the shared ones
  int window, keep;
  float scale;
  ScoreArgs mod;            // its gate is one number a head
};

// The 16-byte slots of a key row are rotated within groups of eight, so that
// consecutive rows of one column spread over the banks; those of a value row
// in pieces of four, which a transposing read takes from four rows at once.
template <int SLOTS>
__device__ __forceinline__ int key_turn(int row) {
  return (SLOTS % 16 == 0 ? row : row >> 1) & 7;
}
template <int SLOTS>
__device__ __forceinline__ int value_turn(int row) {
  return (SLOTS % 16 == 0 ? row & 3 : (row >> 1) & 1) << 2;
}

// MOD: 0 plain scores, 1 with a distance bias, 2 with a soft cap (and the bias,
// if there is one); a sink and the gates are handled in all.
template <int DK, int DE, int NP, bool SHARED, int MOD>
__global__ void __launch_bounds__(256, DE <= 128 ? 2 : 1)
attn_tiles_kernel(TilesArgs a) {
  constexpr int NC = DK / 16;        // 16-wide chunks of the key size
  constexpr int NB = DE / 32;        // 32-row blocks of O^T
  constexpr int KP = DK * 2;         // K row pitch (bytes)
  constexpr int CK = DK / 8, CV = DE / 8;  // 16-byte slots of a row
  // two key tiles, rows as in the cache; apart by name, so that a read of one
  // need not wait for the words on their way into the other
  __shared__ __attribute__((aligned(16))) char k0[64 * KP], k1[64 * KP];
  __shared__ __attribute__((aligned(16))) char v0[128 * DE], v1[128 * DE];

  // later tiles of a portion see more keys: they start first
  const int* tl = a.tiles + 4 * (gridDim.y - 1 - blockIdx.y);
  const int seq = tl[0], row0 = tl[1], nrow = tl[2], p0 = tl[3];
  const int h = blockIdx.x, g = h / (a.H / a.G);
  const int* bt = a.bt + (long)seq * a.MB;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int col = lane & 31, hi = lane >> 5;
  const int my = wid * 32 + col;              // query row in the tile
  const int my_pos = p0 + my;
  const int D = a.D, E = a.E;

  frag_u qf[NC];
  {
    const short* src =
        a.q + (long)(row0 + min(my, nrow - 1)) * a.qst + (long)h * D;
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      const int d = c * 16 + hi * 8;
      qf[c].u4 = d < D ? *(const uint4v*)(src + d) : uint4v{0, 0, 0, 0};
    }
  }

  f32x16 ot[NB] = {};
  float m_run = NEG_BIG, l_run = 0.f;
  const float s2 = a.scale * SV_LOG2E *
      (a.mod.temp ? bits2f(((const short*)a.mod.temp)[h]) : 1.f);
  const float slope = MOD && a.mod.slope ? a.mod.slope[h] * SV_LOG2E : 0.f;
  // tanh(x) = 1 - 2 / (1 + e^2x), with x in units of log 2 / cap
  const float cap2 = MOD == 2 ? a.mod.cap * SV_LOG2E : 0.f;
  const float in_cap = MOD == 2 ? 2.f / a.mod.cap : 0.f;

  const int q_hi = p0 + nrow - 1;
  const int t_hi = q_hi / SV_PAGE;
  const int lo = a.window > 0 ? max(0, p0 - a.window + 1) : 0;
  const int nk = a.window > 0
                     ? min((a.keep + SV_PAGE - 1) / SV_PAGE, t_hi + 1) : 0;
  const int t_lo = max(nk, lo / SV_PAGE);
  const int ntiles = nk + max(0, t_hi - t_lo + 1);
  const int w_lo = p0 + wid * 32, w_hi = min(w_lo + 31, q_hi);

  // 32-bit within a page
  const int krow = (int)a.krow, vrow = (int)a.vrow, rrow = (int)a.rrow;
  auto tile_of = [&](int n) { return n < nk ? n : t_lo + n - nk; };
  // Ask for the rows of a tile: a wave's 64 slots of 16 bytes follow each
  // other in LDS, so the rotation of a row's slots is done on the source.
  auto issue = [&](int n, char* kd, char* vd) {
    const long page = bt[tile_of(n)];
    const short* kb = a.kc + page * a.kpage + g * a.khead;
    const short* vb = a.vc + page * a.vpage + g * a.vhead;
    const short* rb = SHARED ? a.kr + page * SV_PAGE * rrow - a.DS : nullptr;
#pragma unroll
    for (int p = 0; p < CK / 4; ++p) {
      const int it = p * 256 + tid, r = it / CK;
      const int c = (it % CK ^ key_turn<CK>(r)) * 8;
      if (c >= D) continue;
      __builtin_amdgcn_global_load_lds(
          (global_ptr)(SHARED && c >= a.DS ? rb + (r * rrow + c)
                                           : kb + (r * krow + c)),
          (lds_ptr)(kd + (p * 256 + wid * 64) * 16), 16, 0, 0);
    }
#pragma unroll
    for (int p = 0; p < CV / 4; ++p) {
      const int it = p * 256 + tid, r = it / CV;
      const int c = (it % CV ^ value_turn<CV>(r)) * 8;
      if (c >= E) continue;
      __builtin_amdgcn_global_load_lds(
          (global_ptr)(vb + (r * vrow + c)),
          (lds_ptr)(vd + (p * 256 + wid * 64) * 16), 16, 0, 0);
    }
  };
  // this lane's part of the addresses in a tile (bytes): slot 2 c + hi of key
  // row col; a transposing read, where 16 lanes turn 4 keys by 16 columns
  int kx[4];
#pragma unroll
  for (int c = 0; c < 4; ++c)
    kx[c] = col * KP + ((2 * c + hi) ^ key_turn<CK>(col)) * 16;
  const int tr_key = 4 * hi + ((lane & 15) >> 2);
  const int vx = (tr_key * DE + ((lane >> 4) & 1) * 16 + (lane & 3) * 4 +
                  value_turn<CV>(tr_key) * 8) * 2;

  auto attend = [&](int n, const char* kbuf, char* vbuf) {
    const int kv0 = tile_of(n) * SV_PAGE;
    const bool active = wid * 32 < nrow && kv0 <= w_hi &&
        (a.window <= 0 || kv0 < a.keep || kv0 + SV_PAGE - 1 > w_lo - a.window);
    if (!active) return;

    f32x16 acc[2] = {};
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int kb = 0; kb < 2; ++kb) {
        frag_u kf;
        kf.u4 = *(const uint4v*)(kbuf + kx[c & 3] + (c >> 2) * 128 +
                                 kb * 32 * KP);
        acc[kb] = mfma_bf16(kf.bf, qf[c].bf, acc[kb]);
      }
    // the reads run two chunks ahead
    __builtin_amdgcn_sched_group_barrier(0x100, 4, 0);
#pragma unroll
    for (int c = 0; c < NC - 2; ++c) {
      __builtin_amdgcn_sched_group_barrier(0x8, 2, 0);
      __builtin_amdgcn_sched_group_barrier(0x100, 2, 0);
    }
    __builtin_amdgcn_sched_group_barrier(0x8, 4, 0);

    const bool masked = kv0 + SV_PAGE - 1 > w_lo ||
        (a.window > 0 && w_hi - kv0 >= a.window &&
         kv0 + SV_PAGE > a.keep);
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) acc[kb] *= s2;
    const int i0 = my_pos - kv0;               // keys up to i0 are not ahead
    if (MOD == 2)
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int r = 0; r < 16; ++r)
          acc[kb][r] = cap2 - 2.f * cap2 * __builtin_amdgcn_rcpf(
              1.f + __builtin_amdgcn_exp2f(acc[kb][r] * in_cap));
    if (MOD == 1 || (MOD == 2 && slope != 0.f))
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int r = 0; r < 16; ++r)
          acc[kb][r] -= slope * (float)(i0 - 32 * kb - acc_row(r, hi));
    if (masked) {
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int j = 32 * kb + acc_row(r, hi);
          const bool gone = j > i0 || (a.window > 0 && i0 - j >= a.window &&
                                       kv0 + j >= a.keep);
          acc[kb][r] = gone ? NEG_BIG : acc[kb][r];
        }
    }
    float mt = NEG_BIG;
#pragma unroll
    for (int kb = 0; kb < 2; ++kb)
#pragma unroll
      for (int r = 0; r < 16; ++r) mt = fmaxf(mt, acc[kb][r]);
    mt = fmaxf(mt, __shfl_xor(mt, 32, 64));
    const float m_new = fmaxf(m_run, mt);
    const float m_eff = fmaxf(m_new, -1e28f);  // an all-masked row stays 0
    const float alpha = __builtin_amdgcn_exp2f(m_run - m_eff);
    m_run = m_new;
    float ps = 0.f;
#pragma unroll
    for (int kb = 0; kb < 2; ++kb)
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        acc[kb][r] = __builtin_amdgcn_exp2f(acc[kb][r] - m_eff);
        ps += acc[kb][r];
      }
    ps += __shfl_xor(ps, 32, 64);
    l_run = l_run * alpha + ps;
    if (__ballot(alpha != 1.f)) {
#pragma unroll
      for (int nb = 0; nb < NB; ++nb) ot[nb] *= alpha;
    }

#pragma unroll
    for (int kb = 0; kb < 2; ++kb)
#pragma unroll
      for (int cc = 0; cc < 2; ++cc) {
        frag_u pf[NP];
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          float x = acc[kb][8 * cc + 2 * u], y = acc[kb][8 * cc + 2 * u + 1];
#pragma unroll
          for (int z = 0; z < NP; ++z) {
            const uint w = pack_bf16x2(x, y);
            pf[z].u[u] = w;
            x -= __uint_as_float(w << 16);
            y -= __uint_as_float(w & 0xffff0000u);
          }
        }
#pragma unroll
        for (int nb = 0; nb < NB; ++nb) {
          union { tr4 t[2]; bf16x8 bf; } vf;
#pragma unroll
          for (int u = 0; u < 2; ++u)
            vf.t[u] = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
                (lds_tr4)(vbuf + (vx ^ (nb * 64)) +
                          (32 * kb + 16 * cc + 8 * u) * DE * 2));
#pragma unroll
          for (int z = 0; z < NP; ++z)
            ot[nb] = mfma_bf16(vf.bf, pf[z].bf, ot[nb]);
        }
        __builtin_amdgcn_sched_group_barrier(0x100, 4, 0);
#pragma unroll
        for (int nb = 0; nb < NB - 2; ++nb) {
          __builtin_amdgcn_sched_group_barrier(0x8, NP, 0);
          __builtin_amdgcn_sched_group_barrier(0x100, 2, 0);
        }
        __builtin_amdgcn_sched_group_barrier(0x8, 2 * NP, 0);
      }
  };

  if (D < DK) {                // columns that no tile writes
    for (int i = tid; i < 64 * CK; i += 256) {
      *(uint4v*)(k0 + i * 16) = uint4v{0, 0, 0, 0};
      *(uint4v*)(k1 + i * 16) = uint4v{0, 0, 0, 0};
    }
    __syncthreads();
  }
  issue(0, k0, v0);
  __syncthreads();             // also waits for the words on their way
  for (int n = 0; n < ntiles; n += 2) {
    const bool more = n + 1 < ntiles;
    if (more) issue(n + 1, k1, v1);
    attend(n, k0, v0);
    __syncthreads();
    if (!more) break;
    if (n + 2 < ntiles) issue(n + 2, k0, v0);
    attend(n + 1, k1, v1);
    __syncthreads();
  }

  if (my >= nrow) return;
  float inv = 1.f / l_run;
  if (a.mod.sink) {
    const float sink = bits2f(((const short*)a.mod.sink)[h]) * SV_LOG2E;
    const float mn = fmaxf(m_run, sink);
    const float c = __builtin_amdgcn_exp2f(m_run - mn);
    inv = c / (l_run * c + __builtin_amdgcn_exp2f(sink - mn));
  }
  if (a.mod.gate)
    inv *= sigmoid_f(bits2f(
        ((const short*)a.mod.gate)[(long)(row0 + my) * a.mod.gst + h]));
  short* dst = a.out + ((long)(row0 + my) * a.H + h) * E;
#pragma unroll
  for (int nb = 0; nb < NB; ++nb)
#pragma unroll
    for (int rg = 0; rg < 4; ++rg) {
      const int d = 32 * nb + 8 * rg + 4 * hi;
      if (d < E) {
        float o[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) o[j] = ot[nb][4 * rg + j] * inv;
        if (a.gate) {
          float z[4];
          load4(a.gate + (long)(row0 + my) * a.gst + (long)h * E + d, z);
#pragma unroll
          for (int j = 0; j < 4; ++j) o[j] *= sigmoid_f(z[j]);
        }
        uint2 w = {pack_bf16x2(o[0], o[1]), pack_bf16x2(o[2], o[3])};
        *(uint2*)(dst + d) = w;
      }
    }
}

// D, DS and E multiples of 8, at most 256; every row 16-byte aligned
extern "C" int sv_attn_tiles(const TilesArgs* a, int n_tiles,
                             hipStream_t stream) {
  if (n_tiles <= 0) return 0;
  const dim3 grid(a->H, n_tiles);
  const int mod = a->mod.cap > 0.f ? 2 : a->mod.slope ? 1 : 0;
  if (a->kr && mod) return 1;
#define ATK(K, V, S, M) \
  attn_tiles_kernel<K, V, 3, S, M><<<grid, 256, 0, stream>>>(*a)
#define AT(K, V)                          \
  do {                                    \
    if (a->kr) ATK(K, V, true, 0);        \
    else if (mod == 2) ATK(K, V, false, 2); \
    else if (mod == 1) ATK(K, V, false, 1); \
    else ATK(K, V, false, 0);             \
  } while (0)
  if (a->D <= 64 && a->E <= 64) AT(64, 64);
  else if (a->D <= 128 && a->E <= 128) AT(128, 128);
  else if (a->D <= 192 && a->E <= 128) AT(192, 128);
  else if (a->D <= 256 && a->E <= 256) AT(256, 256);
  else return 1;
#undef AT
#undef ATK
  return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// rotary embedding (rotate-half) of the rows of a ragged batch, in place:
// every row has its own position.  cos/sin [positions][D / 2] f32.
// ---------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256)
rope_rows_kernel(T* __restrict__ q, long qst, int H, T* __restrict__ k,
                 long kst, int G, const float* __restrict__ cosp,
                 const float* __restrict__ sinp, const int* __restrict__ pos,
                 int D) {
  const int t = blockIdx.x, half = D / 2;
  const long at = (long)pos[t] * half;
  for (int i = threadIdx.x; i < (H + G) * half; i += 256) {
    const int h = i / half, j = i % half;
    T* p = h < H ? q + t * qst + (long)h * D : k + t * kst + (long)(h - H) * D;
    const float c = cosp[at + j], s = sinp[at + j];
    const float x = to_f(p[j]), y = to_f(p[j + half]);
    from_f(p[j], x * c - y * s);
    from_f(p[j + half], y * c + x * s);
  }
}

extern "C" int sv_rope_rows(void* q, long qst, int H, void* k, long kst,
                            int G, const float* cosp, const float* sinp,
                            const int* pos, int T, int D, int f32,
                            hipStream_t stream) {
  if (T <= 0) return 0;
  if (f32)
    rope_rows_kernel<float><<<T, 256, 0, stream>>>(
        (float*)q, qst, H, (float*)k, kst, G, cosp, sinp, pos, D);
  else
    rope_rows_kernel<short><<<T, 256, 0, stream>>>(
        (short*)q, qst, H, (short*)k, kst, G, cosp, sinp, pos, D);
  return (int)hipGetLastError();
}
