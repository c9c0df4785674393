// Mixture of experts for ragged batches: routing, grouping and the grouped
// matrix products.  Every launch has a size that the host knows from the
// number of rows alone, so a decode step can be captured in a graph.
//
//   sv_moe_plan    logits -> chosen experts and weights of each row; (row,
//                  choice) pairs grouped by expert: order and tiles
//   sv_moe_gemm    one grouped product: gate/up with the gated activation in
//                  its epilogue, or down
//
// A pair is row * top + choice.  The order lists the pairs expert by expert;
// a slot is a place in it.  Gate/up reads row pair / top and writes its slot,
// down reads the slot and writes the pair; the weighted sum over a row's
// pairs is taken by the residual norm.

#include "serving.h"

#define MOE_MAX_EXPERTS 512

// ---------------------------------------------------------------------------
// route and plan
// ---------------------------------------------------------------------------
struct MoePlanArgs {
  const float* z;           // [T][E] logits
  const void* bias;         // [E] or null
  int* idx;                 // [T * top] chosen experts
  float* coef;              // [T * top] their weights
  int* order;               // [T * top] slot -> pair
  int* tiles;               // [max_tiles][4]: expert, first slot, slots, 0
  int T, E, top, tile_rows, max_tiles;
  int kind;                 // 0: weights are a softmax over the chosen;
                            // 1: scores sigmoid(z), chosen by score + bias;
                            // 2: weights are a softmax over all experts
  int groups, keep;         // experts of the best groups only (groups > 1)
  int best;                 // a group counts the sum of its 1 or 2 largest
};

// Keep the choice scores v of the best groups of neighbours, drop the others.
// `mem` is the wave's own.
template <int NV>
__device__ __forceinline__ void best_groups(const MoePlanArgs& a, float* v,
                                            float* mem) {
  const int lane = threadIdx.x & 63, size = a.E / a.groups;
#pragma unroll
  for (int i = 0; i < NV; ++i) mem[i * 64 + lane] = v[i];
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
  float score = -INFINITY;
  if (lane < a.groups) {
    float m1 = -INFINITY, m2 = -INFINITY;
    for (int j = 0; j < size; ++j) {
      const float x = mem[lane * size + j];
      m2 = fmaxf(m2, fminf(m1, x));
      m1 = fmaxf(m1, x);
    }
    score = size > 1 && a.best > 1 ? m1 + m2 : m1;
  }
  __builtin_amdgcn_wave_barrier();
  unsigned long long kept = 0;
  for (int k = 0; k < a.keep; ++k) {
    const bool open = lane < a.groups && !(kept >> lane & 1);
    float best = open ? score : -INFINITY;
    int at = open ? lane : 64;
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) {
      const float ob = __shfl_xor(best, off, 64);
      const int oa = __shfl_xor(at, off, 64);
      if (ob > best || (ob == best && oa < at)) {
        best = ob;
        at = oa;
      }
    }
    kept |= 1ull << (at & 63);
  }
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int e = i * 64 + lane;
    if (e < a.E && !(kept >> (e / size) & 1)) v[i] = -INFINITY;
  }
}

// One wave, one row: the largest choice scores in descending order, the lower
// index first among equals.  Choice scores are the logits with their bias, the
// weights a softmax over the chosen, or over all (then they are not scaled to
// a sum of one); or sigmoids with a bias, the weights the chosen sigmoids over
// their sum.
template <typename T>
__device__ __forceinline__ void route_row(const MoePlanArgs& a, int t,
                                          float* mem) {
  const int lane = threadIdx.x & 63;
  constexpr int NV = MOE_MAX_EXPERTS / 64;
  const T* bias = (const T*)a.bias;
  float v[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int e = i * 64 + lane;
    v[i] = -INFINITY;
    if (e < a.E) {
      const float z = a.z[(long)t * a.E + e];
      v[i] = (a.kind == 1 ? 1.f / (1.f + expf(-z)) : z) +
             (bias ? to_f(bias[e]) : 0.f);
    }
  }
  float first = 0.f, sum = 0.f;
  if (a.kind == 2) {            // the softmax's denominator
    first = -INFINITY;
#pragma unroll
    for (int i = 0; i < NV; ++i) first = fmaxf(first, v[i]);
    first = wave_reduce(first, MaxOp());
#pragma unroll
    for (int i = 0; i < NV; ++i) sum += expf(v[i] - first);
    sum = wave_reduce(sum, SumOp());
  }
  if (a.groups > 1) best_groups<NV>(a, v, mem);
  float mine = 0.f;
  int mine_e = 0;
  for (int k = 0; k < a.top; ++k) {
    float best = -INFINITY;
    int at = MOE_MAX_EXPERTS;
#pragma unroll
    for (int i = 0; i < NV; ++i)
      if (v[i] > best) {
        best = v[i];
        at = i * 64 + lane;
      }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) {
      const float ob = __shfl_xor(best, off, 64);
      const int oa = __shfl_xor(at, off, 64);
      if (ob > best || (ob == best && oa < at)) {
        best = ob;
        at = oa;
      }
    }
    at = min(at, a.E - 1);       // logits that are no numbers stay in bounds
#pragma unroll
    for (int i = 0; i < NV; ++i)
      if (at == i * 64 + lane) v[i] = -INFINITY;
    if (k == 0 && a.kind != 2) first = best;
    const float w =
        a.kind == 1 ? 1.f / (1.f + expf(-a.z[(long)t * a.E + at]))
                       : expf(best - first);
    if (a.kind != 2) sum += w;
    if (lane == k) {
      mine = w;
      mine_e = at;
    }
  }
  if (a.kind == 1) sum += 1e-20f;
  if (lane < a.top) {
    a.idx[(long)t * a.top + lane] = mine_e;
    a.coef[(long)t * a.top + lane] = mine / sum;
  }
}

template <typename T>
__global__ void __launch_bounds__(256) moe_route_kernel(MoePlanArgs a) {
  __shared__ float mem[4][MOE_MAX_EXPERTS];
  const int wid = threadIdx.x >> 6, t = blockIdx.x * 4 + wid;
  if (t < a.T) route_row<T>(a, t, mem[wid]);
}

// One workgroup.  ROUTE: it also routes the (few) rows first.
template <typename T, bool ROUTE>
__global__ void __launch_bounds__(1024) moe_plan_kernel(MoePlanArgs a) {
  __shared__ int count[MOE_MAX_EXPERTS], slots[1024], tile_at[1024];
  const int tid = threadIdx.x, E = a.E, pairs = a.T * a.top;
  __shared__ float mem[ROUTE ? 16 : 1][MOE_MAX_EXPERTS];
  if (ROUTE)
    for (int t = tid >> 6; t < a.T; t += 16) route_row<T>(a, t, mem[tid >> 6]);
  for (int e = tid; e < E; e += 1024) count[e] = 0;
  __syncthreads();               // orders the block's own global writes too
  for (int p = tid; p < pairs; p += 1024) atomicAdd(&count[a.idx[p]], 1);
  __syncthreads();
  const int n = tid < E ? count[tid] : 0;
  const int nt = (n + a.tile_rows - 1) / a.tile_rows;
  slots[tid] = n;
  tile_at[tid] = nt;
  __syncthreads();
  for (int off = 1; off < E; off <<= 1) {   // inclusive sums
    const int x = tid >= off ? slots[tid - off] : 0;
    const int y = tid >= off ? tile_at[tid - off] : 0;
    __syncthreads();
    slots[tid] += x;
    tile_at[tid] += y;
    __syncthreads();
  }
  const int total = tile_at[E - 1];
  const int s0 = slots[tid] - n, t0 = tile_at[tid] - nt;
  if (tid < E) {
    for (int i = 0; i < nt; ++i) {
      int* t = a.tiles + 4L * (t0 + i);
      t[0] = tid;
      t[1] = s0 + i * a.tile_rows;
      t[2] = min(a.tile_rows, n - i * a.tile_rows);
      t[3] = 0;
    }
    count[tid] = s0;
  }
  for (int i = total + tid; i < a.max_tiles; i += 1024) a.tiles[4L * i + 2] = 0;
  __syncthreads();
  for (int p = tid; p < pairs; p += 1024)
    a.order[atomicAdd(&count[a.idx[p]], 1)] = p;
}

extern "C" int sv_moe_plan(const MoePlanArgs* a, int f32,
                           hipStream_t stream) {
  if (a->T <= 0) return 0;
  if (a->E > MOE_MAX_EXPERTS || a->top > 64 || a->top > a->E) return 1;
  if (a->groups < 1 || a->groups > 64 || a->E % a->groups || a->keep < 1 ||
      a->keep > a->groups || a->keep * (a->E / a->groups) < a->top ||
      a->best < 1 || a->best > 2)
    return 1;
  const bool fused = a->T <= 64;
  if (!fused) {
    const int grid = (a->T + 3) / 4;
    if (f32) moe_route_kernel<float><<<grid, 256, 0, stream>>>(*a);
    else moe_route_kernel<short><<<grid, 256, 0, stream>>>(*a);
    moe_plan_kernel<float, false><<<1, 1024, 0, stream>>>(*a);
  } else if (f32) {
    moe_plan_kernel<float, true><<<1, 1024, 0, stream>>>(*a);
  } else {
    moe_plan_kernel<short, true><<<1, 1024, 0, stream>>>(*a);
  }
  return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// grouped products
// ---------------------------------------------------------------------------
struct MoeGemmArgs {
  const void* x;            // rows of K
  long xst;
  const void* w;            // [E][2 N or N][K]: gate rows, then up rows
  void* out;                // rows of N
  const int *order, *tiles;
  int top;                  // > 0: x row = pair / top, out row = slot
                            // 0:   x row = slot,       out row = pair
  int N, K, max_tiles;
  float alpha, limit, shift;  // of the gated activation
};

// min(g, limit) sigmoid(alpha g) (clamp(u, +-limit) + shift)
__device__ __forceinline__ float glu(const MoeGemmArgs& a, float g, float u) {
  g = fminf(g, a.limit);
  u = fminf(fmaxf(u, -a.limit), a.limit);
  return g * sigmoid_f(a.alpha * g) * (u + a.shift);
}

// -- MFMA tiles ---------------------------------------
// BM slots x BN weight rows, K in steps of 64 through two LDS buffers; the
// next step's words travel while this one is multiplied: straight into LDS
// (DMA, K a multiple of 64) or through registers.  With a gated activation
// the weight rows of a tile alternate 32 gate, 32 up, so a lane holds both of
// a column.
template <int BM, int BN, int WM, int WN, bool GLU, bool DMA>
__global__ void __launch_bounds__(BM / WM * BN / WN * 64)
moe_tiles_kernel(MoeGemmArgs a) {
  constexpr int NT = BM / WM * BN / WN * 64;
  constexpr int CM = WM / 32, CN = WN / 32;
  constexpr int LX = BM * 8 / NT, LW = BN * 8 / NT;
  constexpr int GROUP = 8;
  constexpr int NOUT = GLU ? BN / 2 : BN;    // columns of a tile's result
  // apart by name, so that a read of one buffer need not wait for the words
  // on their way into the other
  __shared__ __attribute__((aligned(16))) short xs0[BM * 64], xs1[BM * 64];
  __shared__ __attribute__((aligned(16))) short ws0[BN * 64], ws1[BN * 64];

  // neighbours in the list of tiles run on one XCD: groups of GROUP slot
  // tiles by all column tiles, slot tiles fastest
  const int total = gridDim.x;
  int id = blockIdx.x;
  {
    const int per = total / 8, rest = total % 8, xcd = id % 8;
    id = xcd * per + min(xcd, rest) + id / 8;
  }
  const int ntn = (a.N + NOUT - 1) / NOUT;
  const int g0 = id / (GROUP * ntn) * GROUP;
  const int gm = min(GROUP, a.max_tiles - g0);
  const int in = id - g0 * ntn;
  const int tn = in / gm;
  const int* tl = a.tiles + 4L * (g0 + in % gm);
  const int rows = tl[2];
  if (rows == 0) return;
  const int e = tl[0], slot0 = tl[1];

  const int tid = threadIdx.x, lane = tid & 63;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int col = lane & 31, hi = lane >> 5;
  const int wm = wid % (BM / WM) * WM, wn = wid / (BM / WM) * WN;
  const int K = a.K, N = a.N;
  // 16-byte slot (r, s) of a tile lies at place s ^ (r >> 1); thread tid
  // fills places tid, tid + NT, ... of a buffer, NT / 8 rows apart
  const int kc = ((tid ^ (tid >> 4)) & 7) * 8;

  const short* px[LX];
  const short* pw[LW];
#pragma unroll
  for (int i = 0; i < LX; ++i) {
    const int r = (i * NT + tid) / 8;
    const int s = slot0 + min(r, rows - 1);
    px[i] = (const short*)a.x + (long)(a.top ? a.order[s] / a.top : s) * a.xst + kc;
  }
#pragma unroll
  for (int i = 0; i < LW; ++i) {
    const int r = (i * NT + tid) / 8;
    int n = GLU ? tn * NOUT + (r >> 6) * 32 + (r & 31) : tn * NOUT + r;
    n = min(n, N - 1);
    if (GLU && (r & 32)) n += N;
    pw[i] = (const short*)a.w + ((long)e * (GLU ? 2 * N : N) + n) * K + kc;
  }

  uint4v rx[LX], rw[LW];
  auto issue = [&](int k0, short* xs, short* ws) {
    if (DMA) {
      // a wave's 64 places follow each other
#pragma unroll
      for (int i = 0; i < LX; ++i)
        __builtin_amdgcn_global_load_lds(
            (global_ptr)(px[i] + k0), (lds_ptr)(xs + (i * NT + wid * 64) * 8),
            16, 0, 0);
#pragma unroll
      for (int i = 0; i < LW; ++i)
        __builtin_amdgcn_global_load_lds(
            (global_ptr)(pw[i] + k0), (lds_ptr)(ws + (i * NT + wid * 64) * 8),
            16, 0, 0);
      return;
    }
    const bool in_k = k0 + kc < K;
    const uint4v zero = {0, 0, 0, 0};
#pragma unroll
    for (int i = 0; i < LX; ++i) rx[i] = in_k ? *(const uint4v*)(px[i] + k0) : zero;
#pragma unroll
    for (int i = 0; i < LW; ++i) rw[i] = in_k ? *(const uint4v*)(pw[i] + k0) : zero;
  };
  auto commit = [&](short* xs, short* ws) {
    if (DMA) return;
#pragma unroll
    for (int i = 0; i < LX; ++i) *(uint4v*)(xs + (i * NT + tid) * 8) = rx[i];
#pragma unroll
    for (int i = 0; i < LW; ++i) *(uint4v*)(ws + (i * NT + tid) * 8) = rw[i];
  };

  // A step has four chunks of 16 columns.  The fragments of a chunk are read
  // while the one before is multiplied; the last chunk of a step is
  // multiplied after the barrier, while the next step's first is read.
  f32x16 acc[CN][CM] = {};
  frag_u fx[2][CM] = {}, fw[2][CN] = {};
  auto multiply = [&](int c) {
#pragma unroll
    for (int n = 0; n < CN; ++n)
#pragma unroll
      for (int m = 0; m < CM; ++m)
        acc[n][m] = mfma_bf16(fw[c & 1][n].bf, fx[c & 1][m].bf, acc[n][m]);
  };
  auto step = [&](const short* xs, const short* ws) {
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      // row 32 m + col, slot 2 c + hi
      const int at = col * 64 + (((2 * c + hi) ^ (col >> 1)) & 7) * 8;
#pragma unroll
      for (int m = 0; m < CM; ++m)
        fx[c & 1][m].u4 = *(const uint4v*)(xs + wm * 64 + at + m * 2048);
#pragma unroll
      for (int n = 0; n < CN; ++n)
        fw[c & 1][n].u4 = *(const uint4v*)(ws + wn * 64 + at + n * 2048);
      multiply(c - 1);             // of the step before, if c is 0
      // two products, the reads, the other products
      __builtin_amdgcn_sched_group_barrier(0x8, CM * CN < 2 ? 1 : 2, 0);
      __builtin_amdgcn_sched_group_barrier(0x100, CM + CN, 0);
      if (CM * CN > 2) __builtin_amdgcn_sched_group_barrier(0x8, CM * CN - 2, 0);
    }
    __builtin_amdgcn_sched_barrier(0);
  };
  const int steps = (K + 63) / 64;
  issue(0, xs0, ws0);
  commit(xs0, ws0);
  __syncthreads();                 // also waits for the words on their way
  for (int i = 0; i + 1 < steps; i += 2) {
    issue(i * 64 + 64, xs1, ws1);
    step(xs0, ws0);
    commit(xs1, ws1);
    __syncthreads();
    issue(min(i + 2, steps - 1) * 64, xs0, ws0);   // the last one is not read
    step(xs1, ws1);
    commit(xs0, ws0);
    __syncthreads();
  }
  if (steps & 1) step(xs0, ws0);
  multiply(3);

#pragma unroll
  for (int m = 0; m < CM; ++m) {
    const int r = wm + 32 * m + col;
    if (r >= rows) continue;
    const long orow = a.top ? slot0 + r : a.order[slot0 + r];
    short* dst = (short*)a.out + orow * N;
#pragma unroll
    for (int n = 0; n < CN; n += GLU ? 2 : 1)
#pragma unroll
      for (int rg = 0; rg < 4; ++rg) {
        const int c = tn * NOUT + (GLU ? wn / 2 + 16 * n : wn + 32 * n) +
                      8 * rg + 4 * hi;
        if (c >= N) continue;
        float v[4];
#pragma unroll
        for (int j = 0; j < 4; ++j)
          v[j] = GLU ? glu(a, acc[n][m][4 * rg + j],
                           acc[n + (GLU ? 1 : 0)][m][4 * rg + j])
                     : acc[n][m][4 * rg + j];
        *(uint2*)(dst + c) = uint2{pack_bf16x2(v[0], v[1]),
                                   pack_bf16x2(v[2], v[3])};
      }
  }
}

// -- a few rows per expert: stream the weights --------------------------------
// One workgroup = 32 weight rows (16 gate and their 16 up rows) by up to 32
// slots; its four waves take every fourth 64-column block of K and meet in
// LDS.  Weights go straight from memory to registers, once per tile.
template <bool GLU>
__global__ void __launch_bounds__(256) moe_stream_kernel(MoeGemmArgs a) {
  constexpr int NOUT = GLU ? 16 : 32;
  __shared__ float part[4][16][64];
  const int* tl = a.tiles + 4L * blockIdx.y;
  const int rows = tl[2];
  if (rows == 0) return;
  const int e = tl[0], slot0 = tl[1];
  const int lane = threadIdx.x & 63;
  const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int col = lane & 31, hi = lane >> 5;
  const int K = a.K, N = a.N, n0 = blockIdx.x * NOUT;
  const int n = min(n0 + (GLU ? col & 15 : col), N - 1);
  const bool live = col < rows;
  const int slot = slot0 + (live ? col : 0);
  const int pair = a.order[slot];
  const short* w = (const short*)a.w +
      ((long)e * (GLU ? 2 * N : N) + n + (GLU && col >= 16 ? N : 0)) * K + 32 * hi;
  const short* x = (const short*)a.x +
      (long)(a.top ? pair / a.top : slot) * a.xst + 32 * hi;

  f32x16 acc = {};
  const uint4v zero = {0, 0, 0, 0};
  for (int k0 = wid * 64; k0 < K; k0 += 512) {
    frag_u fw[8], fx[8];
#pragma unroll
    for (int c = 0; c < 8; ++c) {
      const int k = k0 + (c >> 2) * 256 + (c & 3) * 8;  // this lane's order
      const bool in = k + 32 * hi < K;
      fw[c].u4 = in ? *(const uint4v*)(w + k) : zero;
      fx[c].u4 = in && live ? *(const uint4v*)(x + k) : zero;
    }
#pragma unroll
    for (int c = 0; c < 8; ++c) acc = mfma_bf16(fw[c].bf, fx[c].bf, acc);
  }
#pragma unroll
  for (int r = 0; r < 16; ++r) part[wid][r][lane] = acc[r];
  __syncthreads();
  auto total = [&](int r) {
    return part[0][r][lane] + part[1][r][lane] + part[2][r][lane] +
           part[3][r][lane];
  };
  if (!live || (GLU && wid >= 2)) return;
  // accumulator rows 4 w .. 4 w + 3 are weight rows 8 w + 4 hi + 0..3
  const int c = n0 + 8 * wid + 4 * hi;
  if (c >= N) return;
  float v[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    v[j] = total(4 * wid + j);
    if (GLU) v[j] = glu(a, v[j], total(8 + 4 * wid + j));
  }
  short* dst = (short*)a.out + (long)(a.top ? slot : pair) * N + c;
  *(uint2*)dst = uint2{pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3])};
}

// -- any size and type -------------------------------------------------------
template <typename T, bool GLU>
__global__ void __launch_bounds__(256) moe_plain_kernel(MoeGemmArgs a) {
  constexpr int B = 32;
  __shared__ float xs[B][B + 1], gs[B][B + 1], us[GLU ? B : 1][B + 1];
  const int* tl = a.tiles + 4L * blockIdx.y;
  const int rows = tl[2];
  if (rows == 0) return;
  const int e = tl[0], slot0 = tl[1], n0 = blockIdx.x * B;
  const int tx = threadIdx.x & 15, ty = threadIdx.x >> 4;
  const int K = a.K, N = a.N;
  const T* w = (const T*)a.w + (long)e * (GLU ? 2 * N : N) * K;
  float g[2][2] = {}, u[2][2] = {};
  for (int k0 = 0; k0 < K; k0 += B) {
    for (int i = threadIdx.x; i < B * B; i += 256) {
      const int r = i / B, k = k0 + i % B;
      const int s = slot0 + r;
      float xv = 0.f, gv = 0.f, uv = 0.f;
      if (k < K) {
        if (r < rows)
          xv = to_f(((const T*)a.x)[(long)(a.top ? a.order[s] / a.top : s) *
                                    a.xst + k]);
        if (n0 + r < N) {
          gv = to_f(w[(long)(n0 + r) * K + k]);
          if (GLU) uv = to_f(w[(long)(N + n0 + r) * K + k]);
        }
      }
      xs[r][i % B] = xv;
      gs[r][i % B] = gv;
      if (GLU) us[r][i % B] = uv;
    }
    __syncthreads();
    for (int k = 0; k < B; ++k)
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) {
          const float xv = xs[ty + 16 * i][k];
          g[i][j] += xv * gs[tx + 16 * j][k];
          if (GLU) u[i][j] += xv * us[tx + 16 * j][k];
        }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int r = ty + 16 * i, c = n0 + tx + 16 * j;
      if (r >= rows || c >= N) continue;
      const long orow = a.top ? slot0 + r : a.order[slot0 + r];
      from_f(((T*)a.out)[orow * N + c], GLU ? glu(a, g[i][j], u[i][j]) : g[i][j]);
    }
}

template <int BM, int BN, int WM, int WN, bool GLU>
static void launch_tiles(const MoeGemmArgs& a, hipStream_t stream) {
  constexpr int NOUT = GLU ? BN / 2 : BN;
  constexpr int NT = BM / WM * BN / WN * 64;
  const long grid = (long)a.max_tiles * ((a.N + NOUT - 1) / NOUT);
  if (a.K % 64 == 0)
    moe_tiles_kernel<BM, BN, WM, WN, GLU, true><<<grid, NT, 0, stream>>>(a);
  else
    moe_tiles_kernel<BM, BN, WM, WN, GLU, false><<<grid, NT, 0, stream>>>(a);
}

// how: 0 any size and type, 1 stream, 2 to 5 tiles (1 to 5: bf16, N, K, xst
// and bases in 8 elements).  The plan's tile_rows: 32, 32, 32, 64, 128, 256.
extern "C" int sv_moe_gemm(const MoeGemmArgs* a, int how, int gated, int f32,
                           hipStream_t stream) {
  if (a->max_tiles <= 0) return 0;
  if (how == 5) {
    if (gated) launch_tiles<256, 256, 128, 64, true>(*a, stream);
    else launch_tiles<256, 256, 128, 64, false>(*a, stream);
  } else if (how == 4) {
    if (gated) launch_tiles<128, 256, 64, 64, true>(*a, stream);
    else launch_tiles<128, 256, 64, 64, false>(*a, stream);
  } else if (how == 3) {
    if (gated) launch_tiles<64, 256, 64, 64, true>(*a, stream);
    else launch_tiles<64, 128, 64, 32, false>(*a, stream);
  } else if (how == 2) {
    if (gated) launch_tiles<32, 256, 32, 64, true>(*a, stream);
    else launch_tiles<32, 128, 32, 32, false>(*a, stream);
  } else if (how == 1) {
    const dim3 grid((a->N + (gated ? 15 : 31)) / (gated ? 16 : 32), a->max_tiles);
    if (gated) moe_stream_kernel<true><<<grid, 256, 0, stream>>>(*a);
    else moe_stream_kernel<false><<<grid, 256, 0, stream>>>(*a);
  } else {
    const dim3 grid((a->N + 31) / 32, a->max_tiles);
#define PK(T, G) moe_plain_kernel<T, G><<<grid, 256, 0, stream>>>(*a)
    if (f32) { if (gated) PK(float, true); else PK(float, false); }
    else     { if (gated) PK(short, true); else PK(short, false); }
#undef PK
  }
  return (int)hipGetLastError();
}
