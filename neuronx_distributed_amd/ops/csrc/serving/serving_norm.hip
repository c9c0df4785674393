// Norms and pointwise steps of the serving path (32-bit residual stream).
//
// residual_norm: one pass that (1) adds a pending sublayer result to the
// 32-bit residual, (2) stores the new residual, (3) writes the row for the
// next projection (RMS-normed, or just rounded) and/or the concatenation
// [x; x0] that a looped block projects.  The pending result is nothing, one
// tensor, a weighted sum of several rows a token (expert outputs), or two
// parallel branches.  One tensor or sum may be RMS-normed before it is added,
// two branches always are; the result is scaled.  A norm may run in groups:
// equal consecutive parts of the row, each over its own root mean square.
// Instead of one result, up to two gated ones may be pending: each a tensor or
// a weighted sum of rows, plus another tensor, times the sigmoid of a gate an
// element.
//
// The normed rows of single tokens may pass a causal convolution over time on
// their way out (h + conv(h)): the last inputs of their request come from a
// ring, which takes the new one.
//
// gated_norm: RMS norm over groups of a row, times a weight if there is one,
// times sigmoid(gate) or silu(gate) if there is one — the output stage of the
// recurrent mixers.

#include "serving.h"

struct BranchArgs {
  const void* delta;     // [rows, W], or [rows * parts, W] with coef
  const float* coef;     // [rows, parts] or null
  const void* plus;      // [rows, W] added to it, or null
  const void* gate;      // [rows] rows of W; sigmoid(gate + bias) multiplies
  long gst;              //   the sum; or null
  const void* bias;      // [W] or null
  long parts;
};

struct ResidualNormArgs {
  const float* x;        // [rows, W] residual, or null (starts from zero)
  const void* delta;     // [rows, W] T (or f32), or null
  const void* delta2;    // second branch, or null
  const void* w1;        // norm weights [W] of the pending result, or null
  const void* w2;        // of the second branch
  const float* coef;     // [rows, parts]: delta is [rows * parts, W]; or null
  const void* vec;       // [W] added to every row, or null
  float* x_out;          // [out_rows, W] or null
  void* h;               // [out_rows, W] normed * w, or null
  const void* w;         // [W] weight of the norm; null: h is x, rounded
  void* cat;             // [out_rows, 2 W]: new x, then x0; or null
  const void* x0;        // [rows, W]
  const int* index;      // out row -> row, or null
  // convolution of the rows from conv_row on, which are single tokens
  const void* conv;      // [taps][W] weights, or null
  void* ring;            // [slots][taps][W]: the input at position p is in
                         //   place p % taps
  const int* singles;    // [][4]: slot, row, 1, position
  void* hc;              // [out_rows, W] convolved rows
  int rows_out, W, delta_f32, parts;
  int groups, p_groups;  // parts of the norm and of the pending result's norm
  int taps, conv_row;
  float eps, scale;
  float w_base, p_base;  // added to w, and to w1 and w2
  float h_scale;         // multiplies h
  int branches;          // gated results that are pending
  BranchArgs br[2];
};

template <typename T, int VEC>
__device__ __forceinline__ void ld(const T* p, float* v) {
  if (VEC == 4) load4(p, v); else v[0] = to_f(p[0]);
}
template <typename T, int VEC>
__device__ __forceinline__ void st(T* p, const float* v) {
  if (VEC == 4) store4(p, v); else from_f(p[0], v[0]);
}

template <typename T, int VEC, bool BRANCHES, int NT>
__global__ void __launch_bounds__(NT)
residual_norm_kernel(ResidualNormArgs a) {
  extern __shared__ __attribute__((aligned(16))) float row[];  // [W]
  float* part_rstd = row + a.W;    // [groups], if a norm has several
  __shared__ float red[16];
  const int o = blockIdx.x;
  const long r = a.index ? a.index[o] : o;
  const int W = a.W, tid = threadIdx.x;
  const T* d1 = (const T*)a.delta + r * W;
  const float* d1f = (const float*)a.delta + r * W;
  const T* d2 = (const T*)a.delta2 + r * W;

  // the pending result when it is one tensor or a weighted sum of rows
  auto single = [&](int i, float* v) {
    if (a.coef) {
      float t[VEC];
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] = 0.f;
      const T* d = (const T*)a.delta + r * a.parts * W;
      for (int p = 0; p < a.parts; ++p) {
        const float c = a.coef[r * a.parts + p];
        ld<T, VEC>(d + (long)p * W + i, t);
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] += c * t[j];
      }
    } else if (a.delta_f32) {
      ld<float, VEC>(d1f + i, v);
    } else {
      ld<T, VEC>(d1 + i, v);
    }
  };

  // 1 / rms of each of n parts of the row in LDS
  auto norm_parts = [&](int n) {
    const int size = W / n, lane = tid & 63;
    __syncthreads();
    for (int g = tid >> 6; g < n; g += NT / 64) {
      float q = 0.f;
      for (int i = lane; i < size; i += 64) q += row[g * size + i] * row[g * size + i];
      q = wave_reduce(q, SumOp());
      if (lane == 0) part_rstd[g] = 1.f / sqrtf(q / size + a.eps);
    }
    __syncthreads();
  };

  float s1 = a.scale, s2 = 0.f;
  if (a.delta2) {
    float q1 = 0.f, q2 = 0.f, v[VEC];
    for (int i = tid * VEC; i < W; i += NT * VEC) {
      ld<T, VEC>(d1 + i, v);
#pragma unroll
      for (int j = 0; j < VEC; ++j) q1 += v[j] * v[j];
      ld<T, VEC>(d2 + i, v);
#pragma unroll
      for (int j = 0; j < VEC; ++j) q2 += v[j] * v[j];
    }
    q1 = block_reduce_sum(q1, red);
    __syncthreads();
    q2 = block_reduce_sum(q2, red);
    __syncthreads();
    s1 = a.scale / sqrtf(q1 / W + a.eps);
    s2 = a.scale / sqrtf(q2 / W + a.eps);
  } else if (a.w1) {
    float q1 = 0.f, v[VEC];
    for (int i = tid * VEC; i < W; i += NT * VEC) {
      single(i, v);
#pragma unroll
      for (int j = 0; j < VEC; ++j) q1 += v[j] * v[j];
      st<float, VEC>(row + i, v);
    }
    if (a.p_groups > 1) {
      norm_parts(a.p_groups);
    } else {
      q1 = block_reduce_sum(q1, red);
      __syncthreads();
      s1 = a.scale / sqrtf(q1 / W + a.eps);
    }
  }
  const int p_size = a.p_groups > 1 ? W / a.p_groups : W;

  float sq = 0.f;
  for (int i = tid * VEC; i < W; i += NT * VEC) {
    float v[VEC], t[VEC], u[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[j] = 0.f;
    if (a.x) ld<float, VEC>(a.x + r * W + i, v);
    if (a.delta2) {
      ld<T, VEC>(d1 + i, t);
      ld<T, VEC>((const T*)a.w1 + i, u);
#pragma unroll
      for (int j = 0; j < VEC; ++j) t[j] *= s1 * (a.p_base + u[j]);
      float p[VEC];
      ld<T, VEC>(d2 + i, p);
      ld<T, VEC>((const T*)a.w2 + i, u);
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] += t[j] + p[j] * s2 * (a.p_base + u[j]);
    } else if (a.w1) {
      ld<float, VEC>(row + i, t);  // written by this same thread
      ld<T, VEC>((const T*)a.w1 + i, u);
      if (a.p_groups > 1) s1 = a.scale * part_rstd[i / p_size];
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] += t[j] * s1 * (a.p_base + u[j]);
    } else if (a.delta) {
      single(i, t);
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] += s1 * t[j];
    }
    if (BRANCHES) {
      // a long workgroup asks for all words first, so that their ways overlap
      constexpr bool AHEAD = NT > 256;
      constexpr int P = AHEAD ? 4 : 2;   // rows of a sum in flight
      float g[2][VEC], e[2][VEC], d[2][P][VEC], q[2][VEC];
      auto fetch = [&](int b) {
        const BranchArgs& z = a.br[b];
        if (z.gate) ld<T, VEC>((const T*)z.gate + r * z.gst + i, g[b]);
        if (z.bias) ld<T, VEC>((const T*)z.bias + i, e[b]);
#pragma unroll
        for (int p = 0; p < P; ++p)
          if (p < z.parts)
            ld<T, VEC>((const T*)z.delta + (r * z.parts + p) * W + i, d[b][p]);
        if (z.plus) ld<T, VEC>((const T*)z.plus + r * W + i, q[b]);
      };
      auto add = [&](int b) {
        const BranchArgs& z = a.br[b];
#pragma unroll
        for (int j = 0; j < VEC; ++j) t[j] = z.plus ? q[b][j] : 0.f;
#pragma unroll
        for (int p = 0; p < P; ++p) {
          if (p >= z.parts) break;
          const float c = z.coef ? z.coef[r * z.parts + p] : 1.f;
#pragma unroll
          for (int j = 0; j < VEC; ++j) t[j] += c * d[b][p][j];
        }
#pragma unroll 2
        for (int p = P; p < z.parts; ++p) {
          const float c = z.coef[r * z.parts + p];
          ld<T, VEC>((const T*)z.delta + (r * z.parts + p) * W + i, u);
#pragma unroll
          for (int j = 0; j < VEC; ++j) t[j] += c * u[j];
        }
#pragma unroll
        for (int j = 0; j < VEC; ++j)
          v[j] += !z.gate ? t[j]
                          : t[j] * sigmoid_f(z.bias ? g[b][j] + e[b][j] : g[b][j]);
      };
      const bool two = a.branches > 1;
      fetch(0);
      if (AHEAD && two) fetch(1);
      add(0);
      if (!AHEAD && two) fetch(1);
      if (two) add(1);
    }
    if (a.vec) {
      ld<T, VEC>((const T*)a.vec + i, t);
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] += t[j];
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) sq += v[j] * v[j];
    if (a.x_out) st<float, VEC>(a.x_out + (long)o * W + i, v);
    if (a.cat) {
      st<T, VEC>((T*)a.cat + 2L * o * W + i, v);
      ld<T, VEC>((const T*)a.x0 + r * W + i, t);
      st<T, VEC>((T*)a.cat + (2L * o + 1) * W + i, t);
    }
    if (a.h) {
      if (a.w) st<float, VEC>(row + i, v);
      else st<T, VEC>((T*)a.h + (long)o * W + i, v);
    }
  }
  if (!a.h || !a.w) return;
  float rstd = 0.f;
  if (a.groups > 1) {
    norm_parts(a.groups);
  } else {
    sq = block_reduce_sum(sq, red);
    rstd = 1.f / sqrtf(sq / W + a.eps);
  }
  const int size = a.groups > 1 ? W / a.groups : W;
  const bool conv = a.conv && o >= a.conv_row;
  const int* sg = a.singles + 4L * (o - a.conv_row);
  for (int i = tid * VEC; i < W; i += NT * VEC) {
    float v[VEC], u[VEC];
    ld<float, VEC>(row + i, v);  // written by this same thread
    ld<T, VEC>((const T*)a.w + i, u);
    if (a.groups > 1) rstd = part_rstd[i / size];
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[j] *= rstd * (a.w_base + u[j]) * a.h_scale;
    if (!conv) {
      st<T, VEC>((T*)a.h + (long)o * W + i, v);
      continue;
    }
    // the ring holds inputs as T, and so enters the row itself
    const int p = sg[3], last = a.taps - 1;
    T* ring = (T*)a.ring + (long)sg[0] * a.taps * W + i;
    const T* cw = (const T*)a.conv + i;
    T h[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      from_f(h[j], v[j]);
      v[j] = to_f(h[j]);
    }
    float acc[VEC];
    ld<T, VEC>(cw + (long)last * W, u);
#pragma unroll
    for (int j = 0; j < VEC; ++j) acc[j] = v[j] + u[j] * v[j];
    for (int k = max(0, last - p); k < last; ++k) {
      float c[VEC];
      ld<T, VEC>(cw + (long)k * W, u);
      ld<T, VEC>(ring + (long)((p - last + k) % a.taps) * W, c);
#pragma unroll
      for (int j = 0; j < VEC; ++j) acc[j] += u[j] * c[j];
    }
    st<T, VEC>(ring + (long)(p % a.taps) * W, v);
    st<T, VEC>((T*)a.hc + (long)o * W + i, acc);
  }
}

extern "C" int sv_residual_norm(const ResidualNormArgs* a, int f32,
                                hipStream_t stream) {
  if (a->rows_out <= 0) return 0;
  const bool staged = (a->h && a->w) || (a->w1 && !a->delta2);
  const int parts = a->groups > a->p_groups ? a->groups : a->p_groups;
  const size_t lds =
      staged ? ((size_t)a->W + (parts > 1 ? parts : 0)) * sizeof(float) : 0;
  if (lds > 160 * 1024 - 256) return 1;
  if (a->W % a->groups || a->W % a->p_groups) return 1;
  if (a->conv && (!a->h || !a->w)) return 1;
  // four elements of a thread lie in one part
  bool vec = a->W % 4 == 0 && (a->W / a->groups) % 4 == 0 &&
             (a->W / a->p_groups) % 4 == 0;
  for (int b = 0; b < a->branches && b < 2; ++b)
    vec = vec && (!a->br[b].gate ||
                  (a->br[b].gst % 4 == 0 &&
                   (size_t)a->br[b].gate % (f32 ? 16 : 8) == 0));
  if (a->branches < 0 || a->branches > 2 || (a->branches && a->delta)) return 1;
  // few rows: a longer workgroup hides the way to memory
  const bool wide = a->rows_out <= 512 && a->W >= 2048;
#define RNB(T, V, B, N)                                                    \
  residual_norm_kernel<T, V, B, N><<<a->rows_out, N, lds, stream>>>(*a)
#define RN(T, V)                                                           \
  do {                                                                     \
    if (a->branches && wide) RNB(T, V, true, 1024);                        \
    else if (a->branches) RNB(T, V, true, 256);                            \
    else RNB(T, V, false, 256);                                            \
  } while (0)
  if (f32) { if (vec) RN(float, 4); else RN(float, 1); }
  else     { if (vec) RN(short, 4); else RN(short, 1); }
#undef RN
#undef RNB
  return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// o [rows, groups * gs] -> o / rms(group) * w * act(gate)
// One wave per (row, group): NW waves of a block take neighbouring groups.
// Long groups take the whole block.
// ---------------------------------------------------------------------------
template <typename T, int VEC, bool BLOCK>
__global__ void __launch_bounds__(256)
gated_norm_kernel(const T* o, const T* __restrict__ w,
                  const T* __restrict__ gate, long gate_stride,
                  T* out, int rows, int groups, int gs,
                  float eps, int silu) {
  __shared__ float red[16];
  const int tid = BLOCK ? threadIdx.x : (threadIdx.x & 63);
  const int step = (BLOCK ? 256 : 64) * VEC;
  const long item = BLOCK ? (long)blockIdx.x
                          : (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= (long)rows * groups) return;  // whole waves leave together
  const long r = item / groups;
  const int off = (int)(item % groups) * gs;
  const T* src = o + item * gs;
  const T* g = gate ? gate + r * gate_stride + off : nullptr;
  float sq = 0.f, v[VEC], u[VEC];
  for (int i = tid * VEC; i < gs; i += step) {
    ld<T, VEC>(src + i, v);
#pragma unroll
    for (int j = 0; j < VEC; ++j) sq += v[j] * v[j];
  }
  sq = BLOCK ? block_reduce_sum(sq, red) : wave_reduce(sq, SumOp());
  const float rstd = 1.f / sqrtf(sq / gs + eps);
  for (int i = tid * VEC; i < gs; i += step) {
    ld<T, VEC>(src + i, v);
#pragma unroll
    for (int j = 0; j < VEC; ++j) u[j] = 1.f;
    if (w) ld<T, VEC>(w + off + i, u);
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[j] *= rstd * u[j];
    if (g) {
      float z[VEC];
      ld<T, VEC>(g + i, z);
#pragma unroll
      for (int j = 0; j < VEC; ++j)
        v[j] *= silu ? z[j] * sigmoid_f(z[j]) : sigmoid_f(z[j]);
    }
    st<T, VEC>(out + item * gs + i, v);
  }
}

extern "C" int sv_gated_norm(const void* o, const void* w, const void* gate,
                             long gate_stride, void* out, int rows,
                             int groups, int gs, float eps, int silu,
                             int vec4, int f32, hipStream_t stream) {
  if (rows <= 0) return 0;
  const bool block = gs > 1024;
  const long items = (long)rows * groups;
  const int grid = (int)(block ? items : (items + 3) / 4);
#define GN(T, V, B)                                                         \
  gated_norm_kernel<T, V, B><<<grid, 256, 0, stream>>>(                     \
      (const T*)o, (const T*)w, (const T*)gate, gate_stride, (T*)out, rows, \
      groups, gs, eps, silu)
#define GNB(T, V) do { if (block) GN(T, V, true); else GN(T, V, false); } while (0)
  if (f32) { if (vec4) GNB(float, 4); else GNB(float, 1); }
  else     { if (vec4) GNB(short, 4); else GNB(short, 1); }
#undef GNB
#undef GN
  return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// pointwise, in place: max(x, 0)^2, the tanh form of gelu;
// cap * tanh(x / cap) (f32)
// ---------------------------------------------------------------------------
struct ReluSquared {
  __device__ static float at(float x) {
    const float p = fmaxf(x, 0.f);
    return p * p;
  }
};
// 0.5 x (1 + tanh(u)) = x sigmoid(2 u)
struct GeluTanh {
  __device__ static float at(float x) {
    const float u = 0.7978845608028654f * (x + 0.044715f * x * x * x);
    return x * sigmoid_f(2.f * u);
  }
};

template <typename T, int VEC, typename F>
__global__ void __launch_bounds__(256)
pointwise_kernel(T* __restrict__ x, long n) {
  const long i = ((long)blockIdx.x * 256 + threadIdx.x) * VEC;
  if (i >= n) return;
  float v[VEC];
  ld<T, VEC>(x + i, v);
#pragma unroll
  for (int j = 0; j < VEC; ++j) v[j] = F::at(v[j]);
  st<T, VEC>(x + i, v);
}

template <typename F>
static int launch_pointwise(void* x, long n, int f32, hipStream_t stream) {
  if (n <= 0) return 0;
  const int vec = n % 4 == 0 ? 4 : 1;
  const long blocks = (n / vec + 255) / 256;
#define PW(T, V) pointwise_kernel<T, V, F><<<blocks, 256, 0, stream>>>((T*)x, n)
  if (f32) { if (vec == 4) PW(float, 4); else PW(float, 1); }
  else     { if (vec == 4) PW(short, 4); else PW(short, 1); }
#undef PW
  return (int)hipGetLastError();
}

extern "C" int sv_relu_squared(void* x, long n, int f32, hipStream_t stream) {
  return launch_pointwise<ReluSquared>(x, n, f32, stream);
}

extern "C" int sv_gelu_tanh(void* x, long n, int f32, hipStream_t stream) {
  return launch_pointwise<GeluTanh>(x, n, f32, stream);
}

// x [rows][n] -> gelu(x) * (columns [at, at + n) of table[token])
template <typename T>
__global__ void __launch_bounds__(256)
gelu_rows_kernel(T* __restrict__ x, const T* __restrict__ table, long tst,
                 const int* __restrict__ tokens, long rows, int n, int at) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= rows * n) return;
  const long r = i / n;
  from_f(x[i], GeluTanh::at(to_f(x[i])) *
                   to_f(table[tokens[r] * tst + at + (int)(i - r * n)]));
}

extern "C" int sv_gelu_rows(void* x, const void* table, long tst,
                            const int* tokens, long rows, int n, int at,
                            int f32, hipStream_t stream) {
  if (rows <= 0) return 0;
  const long blocks = (rows * n + 255) / 256;
  if (f32)
    gelu_rows_kernel<float><<<blocks, 256, 0, stream>>>(
        (float*)x, (const float*)table, tst, tokens, rows, n, at);
  else
    gelu_rows_kernel<short><<<blocks, 256, 0, stream>>>(
        (short*)x, (const short*)table, tst, tokens, rows, n, at);
  return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// polynomial activation over a row z of n values: with N a division by the
// root mean square of the row, out = a N(z) + b N(z^2) + c N(z^3) + e of
// act [4].  One workgroup a row; up to 16384 values stay in registers.
// ---------------------------------------------------------------------------
template <typename T, int VEC>
__global__ void __launch_bounds__(512)
poly_norm_kernel(const T* __restrict__ x, long xst, const T* __restrict__ act,
                 T* __restrict__ out, int n, float eps) {
  constexpr int KEEP = 32 / VEC;
  __shared__ float red[3][8];
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const T* src = x + (long)blockIdx.x * xst;
  T* dst = out + (long)blockIdx.x * n;
  float kept[KEEP][VEC], s[3] = {0.f, 0.f, 0.f};
  auto add = [&](const float* v) {
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      const float q = v[j] * v[j];
      s[0] += q;
      s[1] += q * q;
      s[2] += q * q * q;
    }
  };
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int i = (k * 512 + tid) * VEC;
    if (i < n) ld<T, VEC>(src + i, kept[k]);
  }
#pragma unroll
  for (int k = 0; k < KEEP; ++k)
    if ((k * 512 + tid) * VEC < n) add(kept[k]);
  for (int i = (KEEP * 512 + tid) * VEC; i < n; i += 512 * VEC) {
    float v[VEC];
    ld<T, VEC>(src + i, v);
    add(v);
  }
#pragma unroll
  for (int p = 0; p < 3; ++p) {
    s[p] = wave_reduce(s[p], SumOp());
    if (lane == 0) red[p][wid] = s[p];
  }
  __syncthreads();
  float f[3];
#pragma unroll
  for (int p = 0; p < 3; ++p) {
    float q = 0.f;
#pragma unroll
    for (int w = 0; w < 8; ++w) q += red[p][w];
    f[p] = to_f(act[p]) / sqrtf(q / n + eps);
  }
  const float e = to_f(act[3]);
  auto put = [&](float* v, int i) {
#pragma unroll
    for (int j = 0; j < VEC; ++j)
      v[j] = e + v[j] * (f[0] + v[j] * (f[1] + v[j] * f[2]));
    st<T, VEC>(dst + i, v);
  };
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int i = (k * 512 + tid) * VEC;
    if (i < n) put(kept[k], i);
  }
  for (int i = (KEEP * 512 + tid) * VEC; i < n; i += 512 * VEC) {
    float v[VEC];
    ld<T, VEC>(src + i, v);
    put(v, i);
  }
}

extern "C" int sv_poly_norm(const void* x, long xst, const void* act,
                            void* out, int rows, int n, float eps, int vec4,
                            int f32, hipStream_t stream) {
  if (rows <= 0 || n <= 0) return 0;
#define PN(T, V)                                                            \
  poly_norm_kernel<T, V><<<rows, 512, 0, stream>>>((const T*)x, xst,        \
                                                   (const T*)act, (T*)out, n, eps)
  if (f32) { if (vec4) PN(float, 4); else PN(float, 1); }
  else     { if (vec4) PN(short, 4); else PN(short, 1); }
#undef PN
  return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// x rows of 2 n: gate, then up -> out [rows][n] = silu(gate) up
// ---------------------------------------------------------------------------
template <typename T, int VEC>
__global__ void __launch_bounds__(256)
silu_mul_kernel(const T* __restrict__ x, long xst, T* __restrict__ out,
                int n) {
  const int i = (blockIdx.x * 256 + threadIdx.x) * VEC;
  if (i >= n) return;
  const T* src = x + (long)blockIdx.y * xst + i;
  float g[VEC], u[VEC];
  ld<T, VEC>(src, g);
  ld<T, VEC>(src + n, u);
#pragma unroll
  for (int j = 0; j < VEC; ++j) u[j] *= silu_f(g[j]);
  st<T, VEC>(out + (long)blockIdx.y * n + i, u);
}

extern "C" int sv_silu_mul(const void* x, long xst, void* out, int rows,
                           int n, int vec4, int f32, hipStream_t stream) {
  if (rows <= 0 || n <= 0) return 0;
  for (int r0 = 0; r0 < rows; r0 += 65535) {
    const int part = rows - r0 < 65535 ? rows - r0 : 65535;
#define SM(T, V)                                                           \
  silu_mul_kernel<T, V>                                                    \
      <<<dim3((n / V + 255) / 256, part), 256, 0, stream>>>(               \
          (const T*)x + r0 * xst, xst, (T*)out + (long)r0 * n, n)
    if (f32) { if (vec4) SM(float, 4); else SM(float, 1); }
    else     { if (vec4) SM(short, 4); else SM(short, 1); }
#undef SM
  }
  return (int)hipGetLastError();
}

__global__ void __launch_bounds__(256)
softcap_kernel(float* __restrict__ x, long n, float cap) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i < n) x[i] = cap * tanhf(x[i] / cap);
}

extern "C" int sv_softcap(void* x, long n, float cap, hipStream_t stream) {
  if (n <= 0) return 0;
  softcap_kernel<<<(n + 255) / 256, 256, 0, stream>>>((float*)x, n, cap);
  return (int)hipGetLastError();
}
