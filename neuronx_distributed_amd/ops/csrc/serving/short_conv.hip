// Causal convolution over time, one filter a channel, over the prompt portions
// of a ragged batch:
//
//   y_t = bias + sum_j w[j] x_(t - taps + 1 + j),   out = silu(y), y or x + y
//
// with zeros before the start of a sequence.  A request keeps its last inputs
// in a ring: the input at position p lies in place p % taps, so a single token
// (whose convolution is fused into the kernel that makes or takes its row)
// never writes a place that the same step reads, and an empty context reads
// nothing: a slot needs no clearing when it changes hands.
//
// A thread owns VEC channels of TB rows.  The rows that reach back into the
// ring all belong to the first tile of a portion (taps - 1 <= TB); its threads
// read their channels' places before they write the new ones.

#include "serving.h"

struct ConvArgs {
  const void* x;            // rows of C channels
  long xst;
  const void* w;            // [taps][C]
  const void* bias;         // [C] or null
  void* out;
  long ost;
  void* ring;               // [slots][taps][C]
  const int* seg;           // [][4]: slot, first row, rows, context
  const int* chunks;        // [n_chunks][4]: segment, first row, rows, -
  int n_chunks, chunk, C, taps;
  int silu, add;            // silu(y); x + y
};

template <bool VEC8, typename T, int V>
__device__ __forceinline__ void put(T* p, const float* v) {
  if (VEC8) {
    store4(p, v);
    store4(p + 4, v + 4);
  } else {
#pragma unroll
    for (int j = 0; j < V; ++j) from_f(p[j], v[j]);
  }
}

template <typename T, bool VEC8, int TAPS, int TB>
__global__ void __launch_bounds__(256) short_conv_kernel(ConvArgs a) {
  constexpr int V = VEC8 ? 8 : 1;
  const int sub = (a.chunk + TB - 1) / TB;
  const int* ch = a.chunks + 4 * (blockIdx.x / sub);
  const int skip = blockIdx.x % sub * TB;
  const int n = min(TB, ch[2] - skip);
  const int c = (blockIdx.y * 256 + threadIdx.x) * V;
  if (n <= 0 || c >= a.C) return;
  const int* sg = a.seg + 4 * ch[0];
  const int rows = sg[2], ctx = sg[3], taps = TAPS ? TAPS : a.taps;
  const int row0 = ch[1] + skip, t0 = row0 - sg[1];   // t0: place in the segment
  const T* x = (const T*)a.x + (long)row0 * a.xst + c;
  T* out = (T*)a.out + (long)row0 * a.ost + c;
  T* ring = (T*)a.ring + (long)sg[0] * taps * a.C + c;
  const T* w = (const T*)a.w + c;

  auto read = [&](const T* p, float* v) {
    if (VEC8) load8<true>(p, 8, v);
    else v[0] = to_f(p[0]);
  };
  // the input `t` rows from the first of this tile, t may be negative
  auto input = [&](int t, float* v) {
    const int p = ctx + t0 + t;
    if (t0 + t >= 0) {
      read(x + (long)t * a.xst, v);
    } else if (p >= 0) {
      read(ring + (long)(p % taps) * a.C, v);
    } else {
#pragma unroll
      for (int j = 0; j < V; ++j) v[j] = 0.f;
    }
  };
  float b[V];
#pragma unroll
  for (int j = 0; j < V; ++j) b[j] = 0.f;
  if (a.bias) read((const T*)a.bias + c, b);
  auto finish = [&](int t, const float* cur, float* y) {
#pragma unroll
    for (int j = 0; j < V; ++j) {
      if (a.silu) y[j] = silu_f(y[j]);
      if (a.add) y[j] += cur[j];
    }
    put<VEC8, T, V>(out + (long)t * a.ost, y);
  };

  if (TAPS) {
    constexpr int K = TAPS ? TAPS : 1;
    float wt[K][V], h[K + 3][V];   // h: K - 1 inputs before, four rows
#pragma unroll
    for (int k = 0; k < K; ++k) read(w + (long)k * a.C, wt[k]);
#pragma unroll
    for (int k = 0; k < K - 1; ++k) input(k - (K - 1), h[k]);
    for (int t = 0; t < n; t += 4) {
#pragma unroll
      for (int u = 0; u < 4; ++u)
        read(x + (long)min(t + u, n - 1) * a.xst, h[K - 1 + u]);
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        if (t + u >= n) break;
        float y[V];
#pragma unroll
        for (int j = 0; j < V; ++j) {
          y[j] = b[j];
#pragma unroll
          for (int k = 0; k < K; ++k) y[j] += wt[k][j] * h[u + k][j];
        }
        finish(t + u, h[K - 1 + u], y);
      }
#pragma unroll
      for (int k = 0; k < K - 1; ++k)
#pragma unroll
        for (int j = 0; j < V; ++j) h[k][j] = h[k + 4][j];
    }
  } else {
    for (int t = 0; t < n; ++t) {
      float y[V], v[V], u[V];
#pragma unroll
      for (int j = 0; j < V; ++j) {
        y[j] = b[j];
        v[j] = 0.f;
      }
      for (int k = 0; k < taps; ++k) {
        input(t + k - (taps - 1), v);
        read(w + (long)k * a.C, u);
#pragma unroll
        for (int j = 0; j < V; ++j) y[j] += u[j] * v[j];
      }
      finish(t, v, y);
    }
  }

  if (t0 == 0)                   // after this thread's reads of the ring
    for (int t = max(0, rows - (taps - 1)); t < rows; ++t) {
      float v[V];
      read(x + (long)t * a.xst, v);
      put<VEC8, T, V>(ring + (long)((ctx + t) % taps) * a.C, v);
    }
}

// taps <= 65; vec: C, strides and bases in 8 elements
extern "C" int sv_short_conv(const ConvArgs* a, int vec, int f32,
                             hipStream_t stream) {
  if (a->n_chunks <= 0) return 0;
  if (a->taps < 1 || a->taps > 65) return 1;
  const int per = 256 * (vec ? 8 : 1);
#define SC(T, V, K, B)                                                       \
  short_conv_kernel<T, V, K, B>                                              \
      <<<dim3(a->n_chunks * ((a->chunk + B - 1) / B), (a->C + per - 1) / per), \
         256, 0, stream>>>(*a)
#define SCK(T, V)                              \
  do {                                         \
    if (a->taps == 2) SC(T, V, 2, 16);         \
    else if (a->taps == 3) SC(T, V, 3, 16);    \
    else if (a->taps == 4) SC(T, V, 4, 16);    \
    else SC(T, V, 0, 64);                      \
  } while (0)
  if (f32) { if (vec) SCK(float, true); else SCK(float, false); }
  else     { if (vec) SCK(short, true); else SCK(short, false); }
#undef SCK
#undef SC
  return (int)hipGetLastError();
}
