// Latent attention over a paged cache for ragged batches.
//
// A token keeps one row [latent (R) | rotated shared key (P)] for all heads:
// cache [page][64][R + P].  The key of head h is [W_uk,h c | kr], its value
// W_uv,h c.  Two ways to attend:
//   * absorbed: the query takes W_uk in (q' = W_uk,h^T q), scores and values
//     read the cached rows themselves, W_uv follows; used for single tokens.
//   * expanded: the visible rows are gathered, one GEMM makes keys and values
//     of all heads, and the MFMA prompt kernel of paged_attn.hip runs on them.
//
//   sv_latent_append  norm of the latent, rotation of q and of the shared
//                     key at each row's position, write into the cache
//   sv_latent_gather  cache pages -> contiguous rows
//   sv_head_linear    a small matrix per head (absorption, values), with an
//                     optional sigmoid gate on the result
//   sv_latent_rows    MFMA attention of one absorbed query row over its keys
//
// The denominator of the softmax may hold a sink, a number a head.

#include "serving.h"

#define NEG_BIG (-1e30f)

// ---------------------------------------------------------------------------
// append
// ---------------------------------------------------------------------------
struct LatentAppendArgs {
  void* q;                  // [T] rows; head h's rotated part at h * qh
  long qst, qh;
  void* qr;                 // rotated queries go here (may be q itself)
  long qrst, qrh;
  const void* kv;           // [T] rows of R latents, then P key columns
  long kvst;
  const void* w;            // [R] weight of the latents' norm
  const double* freq;       // [rot / 2] radians a position
  void* cache;
  const int *pos, *seq, *bt;
  int MB, H, R, P, rot;     // rot <= P columns turn, the rest pass
  float eps;
  float amp;                // multiplies cos and sin
  int pairs;                // columns 2i and 2i + 1 turn, not i and i + rot / 2
};

template <typename T>
__global__ void __launch_bounds__(256)
latent_append_kernel(LatentAppendArgs a) {
  extern __shared__ float cs[];          // cos [rot / 2], sin [rot / 2]
  __shared__ float red[16];
  const int t = blockIdx.x, tid = threadIdx.x;
  const int half = a.rot / 2, R = a.R, P = a.P;
  const int p = a.pos[t];
  for (int i = tid; i < half; i += 256) {
    float c, s;
    turn(a.freq[i], p, &c, &s);
    cs[i] = c * a.amp;
    cs[half + i] = s * a.amp;
  }
  const T* kv = (const T*)a.kv + t * a.kvst;
  float sq = 0.f;
  for (int i = tid; i < R; i += 256) {
    const float v = to_f(kv[i]);
    sq += v * v;
  }
  sq = block_reduce_sum(sq, red);        // its barriers publish cs as well
  const float rstd = 1.f / sqrtf(sq / R + a.eps);
  const long page = a.bt[(long)a.seq[t] * a.MB + p / SV_PAGE];
  T* row = (T*)a.cache + (page * SV_PAGE + p % SV_PAGE) * (R + P);
  for (int i = tid; i < R; i += 256)
    from_f(row[i], to_f(kv[i]) * rstd * to_f(((const T*)a.w)[i]));

  auto rotate = [&](const T* src, T* dst, int i) {   // i in [0, P - half)
    if (i < half) {
      const float c = cs[i], s = cs[half + i];
      const int u = a.pairs ? 2 * i : i, w = a.pairs ? u + 1 : i + half;
      const float x = to_f(src[u]), y = to_f(src[w]);
      from_f(dst[u], x * c - y * s);
      from_f(dst[w], y * c + x * s);
    } else {
      dst[i + half] = src[i + half];
    }
  };
  const int items = P - half;
  for (int i = tid; i < (a.H + 1) * items; i += 256) {
    const int h = i / items, j = i % items;
    if (h == a.H)
      rotate(kv + R, row + R, j);
    else
      rotate((const T*)a.q + t * a.qst + h * a.qh,
             (T*)a.qr + t * a.qrst + h * a.qrh, j);
  }
}

extern "C" int sv_latent_append(const LatentAppendArgs* a, int T, int f32,
                                hipStream_t stream) {
  if (T <= 0) return 0;
  const size_t lds = a->rot * sizeof(float);
  if (f32) latent_append_kernel<float><<<T, 256, lds, stream>>>(*a);
  else latent_append_kernel<short><<<T, 256, lds, stream>>>(*a);
  return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// gather: pages[i] of the cache -> page i of the workspace (16-byte words)
// ---------------------------------------------------------------------------
__global__ void __launch_bounds__(256)
latent_gather_kernel(const uint4v* __restrict__ cache, uint4v* __restrict__ ws,
                     const int* __restrict__ pages, int words) {
  const uint4v* s = cache + (long)pages[blockIdx.x] * words;
  uint4v* d = ws + (long)blockIdx.x * words;
  for (int i = blockIdx.y * 256 + threadIdx.x; i < words; i += gridDim.y * 256)
    d[i] = s[i];
}

extern "C" int sv_latent_gather(const void* cache, void* ws, const int* pages,
                                int n, int page_bytes, hipStream_t stream) {
  if (n <= 0) return 0;
  const int words = page_bytes / 16;
  const dim3 grid(n, (words + 1023) / 1024);
  latent_gather_kernel<<<grid, 256, 0, stream>>>((const uint4v*)cache,
                                                 (uint4v*)ws, pages, words);
  return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// head linear: out[t, h, n] = sum_k x[t, h, k] w[h, n, k]
// ---------------------------------------------------------------------------
struct HeadLinearArgs {
  const void* x;
  long xst, xh;             // elements between rows, between heads
  const void* w;            // [H][N][K]
  void* out;
  long ost, oh;
  const void* gate;         // out is multiplied by sigmoid(gate), or null
  long gst, gh;
  int T, H, N, K;
};

// One wave of a workgroup's four takes every fourth 64-column block of K for
// 32 outputs and 32 rows; the partial sums meet in LDS.  With SPLIT off each
// wave has 32 outputs of its own.  K, strides and bases in 8 elements.
template <bool SPLIT>
__global__ void __launch_bounds__(256)
head_linear_mfma_kernel(HeadLinearArgs a) {
  const int lane = threadIdx.x & 63;
  const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int col = lane & 31, hi = lane >> 5;
  const int h = blockIdx.y, t0 = blockIdx.z * 32;
  const int n0 = (SPLIT ? blockIdx.x : blockIdx.x * 4 + wid) * 32;
  const int K = a.K;
  const bool vn = n0 + col < a.N, vt = t0 + col < a.T;
  const short* w = (const short*)a.w + ((long)h * a.N + (vn ? n0 + col : 0)) * K;
  const short* x = (const short*)a.x + (long)(vt ? t0 + col : 0) * a.xst + h * a.xh;
  f32x16 acc = {};
  const uint4v zero = {0, 0, 0, 0};
  if (n0 < a.N)
    for (int k0 = SPLIT ? wid * 64 : 0; k0 < K; k0 += SPLIT ? 256 : 64) {
      frag_u fw[4], fx[4];
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        const int k = k0 + 32 * hi + 8 * c;   // any order, the same for both
        fw[c].u4 = vn && k < K ? *(const uint4v*)(w + k) : zero;
        fx[c].u4 = vt && k < K ? *(const uint4v*)(x + k) : zero;
      }
#pragma unroll
      for (int c = 0; c < 4; ++c) acc = mfma_bf16(fw[c].bf, fx[c].bf, acc);
    }
  if (SPLIT) {
    __shared__ float part[4][16][64];
#pragma unroll
    for (int r = 0; r < 16; ++r) part[wid][r][lane] = acc[r];
    __syncthreads();
    // wave w finishes accumulator rows 4 w .. 4 w + 3
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      float v = 0.f;
#pragma unroll
      for (int s = 0; s < 4; ++s) v += part[s][4 * wid + j][lane];
      acc[j] = v;
    }
  }
  if (!vt) return;
  const int t = t0 + col;
#pragma unroll
  for (int rg = 0; rg < (SPLIT ? 1 : 4); ++rg) {
    const int n = n0 + 8 * (SPLIT ? wid : rg) + 4 * hi;
    if (n + 3 < a.N) {
      float v[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = acc[4 * rg + j];
      if (a.gate) {
        float z[4];
        load4((const short*)a.gate + t * a.gst + h * a.gh + n, z);
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] *= sigmoid_f(z[j]);
      }
      store4((short*)a.out + t * a.ost + h * a.oh + n, v);
    }
  }
}

// any size and type: one output a thread
template <typename T>
__global__ void __launch_bounds__(256)
head_linear_kernel(HeadLinearArgs a) {
  const int n = blockIdx.y * 256 + threadIdx.x, h = blockIdx.z;
  const long t = blockIdx.x;
  if (n >= a.N) return;
  const T* x = (const T*)a.x + t * a.xst + h * a.xh;
  const T* w = (const T*)a.w + ((long)h * a.N + n) * a.K;
  float v = 0.f;
  for (int k = 0; k < a.K; ++k) v += to_f(x[k]) * to_f(w[k]);
  if (a.gate) v *= sigmoid_f(to_f(((const T*)a.gate)[t * a.gst + h * a.gh + n]));
  from_f(((T*)a.out)[t * a.ost + h * a.oh + n], v);
}

extern "C" int sv_head_linear(const HeadLinearArgs* a, int mfma, int f32,
                              hipStream_t stream) {
  if (a->T <= 0) return 0;
  if (mfma) {
    const int nt = (a->N + 31) / 32, tt = (a->T + 31) / 32;
    if (a->K >= 256)
      head_linear_mfma_kernel<true><<<dim3(nt, a->H, tt), 256, 0, stream>>>(*a);
    else
      head_linear_mfma_kernel<false><<<dim3((nt + 3) / 4, a->H, tt), 256, 0,
                                       stream>>>(*a);
  } else {
    const dim3 grid(a->T, (a->N + 255) / 256, a->H);
    if (f32) head_linear_kernel<float><<<grid, 256, 0, stream>>>(*a);
    else head_linear_kernel<short><<<grid, 256, 0, stream>>>(*a);
  }
  return (int)hipGetLastError();
}

// ---------------------------------------------------------------------------
// rows: MFMA attention of absorbed queries.
//
// One workgroup = 4 waves, one query row, 32 heads, a range of its keys in
// tiles of 32 (half a page, contiguous in the cache).  Per tile:
//   1. S^T = K Q^T, each wave a quarter of the columns; partial sums to LDS
//   2. softmax by all threads (8 lanes a head); the 32-bit weights go to LDS
//      as three bf16 planes that add up to them exactly
//   3. O^T += V^T P^T, each wave a quarter of the latent columns; V^T is the
//      same tile, read through the transposing LDS load
// The columns are padded to EP latents and 64 rotated ones, with zeros.
// ---------------------------------------------------------------------------
struct LatentRowsArgs {
  const short* q;           // [rows][H][R + P]
  const short* cache;
  const int *pos, *seq, *bt;
  float* part;              // [rows][H][splits][R + 2] or null (1 split)
  short* out;               // [rows][H][R]
  int MB, rows, H, R, P, splits, window;
  float scale;
  const short* sink;        // [H] or null
};

template <int EP>
__global__ void __launch_bounds__(256, 2)
latent_rows_kernel(LatentRowsArgs a) {
  constexpr int KP = EP + 64;            // columns of a tile row
  constexpr int CPR = KP / 8;            // 16-byte slots of a row
  constexpr int NCW = KP / 64;           // 16-column chunks of a wave
  constexpr int NB = EP >= 128 ? EP / 128 : 1;  // 32-column blocks of a wave
  constexpr int NL = 32 * CPR / 256;     // 16-byte words a thread loads
  constexpr int SP = 36, PP = 40;        // pitches of S and P
  __shared__ __attribute__((aligned(16))) short kt[32 * KP];
  __shared__ __attribute__((aligned(16))) float sp[4][32 * SP];
  __shared__ __attribute__((aligned(16))) short pp[3][32 * PP];
  __shared__ float corr[32], lsum[32], mrow[32];

  const int split = blockIdx.x % a.splits;
  const int unit = blockIdx.x / a.splits;
  const int nhg = (a.H + 31) / 32;
  const int h0 = unit % nhg * 32, row = unit / nhg;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int col = lane & 31, hi = lane >> 5;
  const int R = a.R, P = a.P, RP = R + P;
  const uint4v zero = {0, 0, 0, 0};

  // column of a slot in a cached row, -1 for padding
  auto column = [&](int slot) {
    const int c = slot * 8;
    return c < EP ? (c < R ? c : -1) : (c - EP < P ? R + c - EP : -1);
  };
  auto swz_slot = [](int r, int slot) {
    return slot ^ (CPR % 16 == 0 ? r & 15 : (r >> 1) & 7);
  };

  frag_u qf[NCW];
  {
    const bool live = h0 + col < a.H;
    const short* src = a.q + ((long)row * a.H + (live ? h0 + col : 0)) * RP;
#pragma unroll
    for (int c = 0; c < NCW; ++c) {
      const int k = column((wid * NCW + c) * 2 + hi);
      qf[c].u4 = live && k >= 0 ? *(const uint4v*)(src + k) : zero;
    }
  }

  const int i_pos = a.pos[row];
  const int* bt = a.bt + (long)a.seq[row] * a.MB;
  const int lo = a.window > 0 ? max(0, i_pos - a.window + 1) : 0;
  const int t_lo = lo / 32, total = i_pos / 32 - t_lo + 1;
  const int per = (total + a.splits - 1) / a.splits;
  const int t0 = t_lo + split * per, t1 = min(t_lo + total, t0 + per);

  uint4v reg[NL];
  auto issue = [&](int t) {
    const short* src = a.cache + ((long)bt[t / 2] * SV_PAGE + (t & 1) * 32) * RP;
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int it = i * 256 + tid;
      const int k = column(it % CPR);
      reg[i] = k >= 0 ? *(const uint4v*)(src + it / CPR * RP + k) : zero;
    }
  };

  f32x16 o[NB] = {};
  const int sh = tid >> 3, sk = tid & 7;   // softmax: head, 4-key group
  float m_run = NEG_BIG, l_run = 0.f;
  if (a.sink && split == 0 && h0 + sh < a.H) {   // once for all splits
    m_run = bits2f(a.sink[h0 + sh]) * SV_LOG2E;
    l_run = 1.f;
  }
  const float s2 = a.scale * SV_LOG2E;
  // transposing reads: a group of 16 lanes turns 4 keys x 16 columns
  const int tr_key = (lane & 15) >> 2, tr_col = ((lane >> 4) & 1) * 16 + (lane & 3) * 4;

  if (t0 < t1) issue(t0);
  for (int t = t0; t < t1; ++t) {
    __syncthreads();               // the previous tile has been read
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int it = i * 256 + tid, r = it / CPR;
      *(uint4v*)(kt + r * KP + swz_slot(r, it % CPR) * 8) = reg[i];
    }
    __syncthreads();
    if (t + 1 < t1) issue(t + 1);

    f32x16 acc = {};
#pragma unroll
    for (int c = 0; c < NCW; ++c) {
      frag_u kf;
      kf.u4 = *(const uint4v*)(kt + col * KP +
                               swz_slot(col, (wid * NCW + c) * 2 + hi) * 8);
      acc = mfma_bf16(kf.bf, qf[c].bf, acc);
    }
#pragma unroll
    for (int rg = 0; rg < 4; ++rg)
      *(f32x4*)(sp[wid] + col * SP + 8 * rg + 4 * hi) =
          f32x4{acc[4 * rg], acc[4 * rg + 1], acc[4 * rg + 2], acc[4 * rg + 3]};
    __syncthreads();

    {
      f32x4 s = *(const f32x4*)(sp[0] + sh * SP + 4 * sk);
#pragma unroll
      for (int w = 1; w < 4; ++w) s += *(const f32x4*)(sp[w] + sh * SP + 4 * sk);
      float mt = NEG_BIG;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int key = t * 32 + 4 * sk + j;
        s[j] = key >= lo && key <= i_pos ? s[j] * s2 : NEG_BIG;
        mt = fmaxf(mt, s[j]);
      }
#pragma unroll
      for (int off = 1; off < 8; off <<= 1) mt = fmaxf(mt, __shfl_xor(mt, off, 64));
      const float mn = fmaxf(m_run, mt);   // every tile holds a visible key
      const float al = __builtin_amdgcn_exp2f(m_run - mn);
      m_run = mn;
      float ps = 0.f;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        s[j] = __builtin_amdgcn_exp2f(s[j] - mn);
        ps += s[j];
      }
#pragma unroll
      for (int off = 1; off < 8; off <<= 1) ps += __shfl_xor(ps, off, 64);
      l_run = l_run * al + ps;
      float x[4] = {s[0], s[1], s[2], s[3]};
#pragma unroll
      for (int z = 0; z < 3; ++z) {
        uint2 w = {pack_bf16x2(x[0], x[1]), pack_bf16x2(x[2], x[3])};
        *(uint2*)(pp[z] + sh * PP + 4 * sk) = w;
        x[0] -= __uint_as_float(w.x << 16);
        x[1] -= __uint_as_float(w.x & 0xffff0000u);
        x[2] -= __uint_as_float(w.y << 16);
        x[3] -= __uint_as_float(w.y & 0xffff0000u);
      }
      if (sk == 0) corr[sh] = al;
    }
    __syncthreads();

    const float al = corr[col];
    if (__ballot(al != 1.f)) {
#pragma unroll
      for (int nb = 0; nb < NB; ++nb) o[nb] *= al;
    }
#pragma unroll
    for (int kc = 0; kc < 2; ++kc) {
      frag_u pf[3];
#pragma unroll
      for (int z = 0; z < 3; ++z)
        pf[z].u4 = *(const uint4v*)(pp[z] + col * PP + kc * 16 + hi * 8);
#pragma unroll
      for (int nb = 0; nb < NB; ++nb) {
        const int e = (wid * NB + nb) * 32;
        if (e >= EP) continue;
        union { tr4 h[2]; bf16x8 bf; } vf;
#pragma unroll
        for (int u = 0; u < 2; ++u) {
          const int r = kc * 16 + hi * 8 + u * 4 + tr_key, c = e + tr_col;
          vf.h[u] = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
              (lds_tr4)(kt + r * KP + swz_slot(r, c >> 3) * 8 + (c & 7)));
        }
#pragma unroll
        for (int z = 0; z < 3; ++z) o[nb] = mfma_bf16(vf.bf, pf[z].bf, o[nb]);
      }
    }
  }

  if (sk == 0) {
    lsum[sh] = l_run;
    mrow[sh] = m_run;
  }
  __syncthreads();
  if (h0 + col >= a.H) return;
  const long rh = (long)row * a.H + h0 + col;
  const float inv = 1.f / lsum[col];
#pragma unroll
  for (int nb = 0; nb < NB; ++nb)
#pragma unroll
    for (int rg = 0; rg < 4; ++rg) {
      const int e = (wid * NB + nb) * 32 + 8 * rg + 4 * hi;
      if (e >= R) continue;
      if (a.splits == 1) {
        const uint2 w = {pack_bf16x2(o[nb][4 * rg] * inv, o[nb][4 * rg + 1] * inv),
                         pack_bf16x2(o[nb][4 * rg + 2] * inv,
                                     o[nb][4 * rg + 3] * inv)};
        *(uint2*)(a.out + rh * R + e) = w;
      } else {
        float* p = a.part + (rh * a.splits + split) * (R + 2) + e;
        *(float2*)p = make_float2(o[nb][4 * rg], o[nb][4 * rg + 1]);
        *(float2*)(p + 2) = make_float2(o[nb][4 * rg + 2], o[nb][4 * rg + 3]);
      }
    }
  if (a.splits > 1 && wid == 0 && hi == 0) {
    float* p = a.part + (rh * a.splits + split) * (R + 2) + R;
    p[0] = mrow[col];
    p[1] = lsum[col];
  }
}

extern "C" int sv_attn_merge(const float* part, void* out, long rows,
                             int splits, int E, int f32, hipStream_t stream);

// R and P multiples of 8, R <= 512, P <= 64, rows 16-byte aligned
extern "C" int sv_latent_rows(const LatentRowsArgs* a, hipStream_t stream) {
  if (a->rows <= 0) return 0;
  const long grid = (long)a->rows * ((a->H + 31) / 32) * a->splits;
#define LR(E) latent_rows_kernel<E><<<grid, 256, 0, stream>>>(*a)
  if (a->P > 64) return 1;
  if (a->R <= 64) LR(64);
  else if (a->R <= 128) LR(128);
  else if (a->R <= 256) LR(256);
  else if (a->R <= 512) LR(512);
  else return 1;
#undef LR
  if (a->splits > 1)
    return sv_attn_merge(a->part, a->out, (long)a->rows * a->H, a->splits,
                         a->R, 0, stream);
  return (int)hipGetLastError();
}
