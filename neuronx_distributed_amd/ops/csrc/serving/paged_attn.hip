// Attention over a paged KV cache for ragged batches.
//
// Cache layout: K [page][kv head][64][D], V [page][kv head][64][E]; a
// request's block table maps position / 64 to a page.  Visibility of key j
// for the query at position i:  j <= i and (i - j < window or j < keep).
// window <= 0 means plain causal.  Sizes D and E need not be equal.
//
//   sv_kv_append   writes the K/V rows of a step into their pages
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
// rows
// ---------------------------------------------------------------------------
struct RowsArgs {
  const void *q, *k, *v;       // row 0 of the step's projections
  long qst, kst, vst;          // row strides (elements)
  void *kc, *vc;               // cache
  const int *pos, *seq, *bt;   // per row: position, sequence; block table
  float* part;                 // [rows][H][splits][E + 2] or null (1 split)
  void* out;                   // [rows][H * E]
  int MB, rows, H, G, D, E, splits, append, window, keep;
  float scale;
};

// LPR lanes own one key row (8 dims each); RC query heads share the row.
template <typename T, int LPR, int RC, bool VEC>
__global__ void __launch_bounds__(256)
attn_rows_kernel(RowsArgs a) {
  constexpr int NR = 64 / LPR;     // key rows of one wave step
  constexpr int DV = LPR * 8;
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
  const int d0 = 8 * hl;
  const int nd = min(8, a.D - d0), ne = min(8, a.E - d0);  // <= 0: no dims
  const int D = a.D, E = a.E;

  const int i_pos = a.pos[row];
  const int* bt = a.bt + (long)a.seq[row] * a.MB;

  float qv[RC][8];
#pragma unroll
  for (int r = 0; r < RC; ++r) {
    const int h = g * rep + min(rc * RC + r, rep - 1);
    load8<VEC>((const T*)a.q + row * a.qst + (long)h * D + d0, nd, qv[r]);
  }
  const float s2 = a.scale * SV_LOG2E;
#pragma unroll
  for (int r = 0; r < RC; ++r)
#pragma unroll
    for (int j = 0; j < 8; ++j) qv[r][j] *= s2;

  const T* kn = (const T*)a.k + row * a.kst + (long)g * D;
  const T* vn = (const T*)a.v + row * a.vst + (long)g * E;
  if (a.append && split == 0 && rc == 0) {
    const long page = bt[i_pos / SV_PAGE];
    const long base = (page * a.G + g) * SV_PAGE + i_pos % SV_PAGE;
    for (int i = threadIdx.x; i < D; i += 256)
      ((T*)a.kc)[base * D + i] = kn[i];
    for (int i = threadIdx.x; i < E; i += 256)
      ((T*)a.vc)[base * E + i] = vn[i];
  }

  // visible keys as one list: the kept first ones, then the window.  With
  // append, the row's own key is handled from registers at the end.
  const int lo = a.window > 0 ? max(0, i_pos - a.window + 1) : 0;
  const int nfirst = min(a.keep, lo);
  const int total = nfirst + (i_pos - lo) + (a.append ? 0 : 1);
  const int per = (total + a.splits - 1) / a.splits;
  const int k0 = split * per, k1 = min(total, k0 + per);

  float m[RC], l[RC], o[RC][8];
#pragma unroll
  for (int r = 0; r < RC; ++r) {
    m[r] = NEG_BIG;
    l[r] = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) o[r][j] = 0.f;
  }

  auto fetch = [&](int idx, float* kf, float* vf) {
    const int j = idx < nfirst ? idx : lo + idx - nfirst;
    const long base =
        ((long)bt[j / SV_PAGE] * a.G + g) * SV_PAGE + j % SV_PAGE;
    load8<VEC>((const T*)a.kc + base * D + d0, nd, kf);
    load8<VEC>((const T*)a.vc + base * E + d0, ne, vf);
  };
  auto absorb = [&](const float* kf, const float* vf, bool live) {
    float s[RC];
#pragma unroll
    for (int r = 0; r < RC; ++r) {
      s[r] = 0.f;
#pragma unroll
      for (int j = 0; j < 8; ++j) s[r] += qv[r][j] * kf[j];
    }
#pragma unroll
    for (int off = LPR / 2; off > 0; off >>= 1)
#pragma unroll
      for (int r = 0; r < RC; ++r) s[r] += __shfl_xor(s[r], off, 64);
#pragma unroll
    for (int r = 0; r < RC; ++r) {
      const float mn = live ? fmaxf(m[r], s[r]) : m[r];
      const float al = __builtin_amdgcn_exp2f(m[r] - mn);
      const float p = live ? __builtin_amdgcn_exp2f(s[r] - mn) : 0.f;
      m[r] = mn;
      l[r] = l[r] * al + p;
#pragma unroll
      for (int j = 0; j < 8; ++j) o[r][j] = o[r][j] * al + p * vf[j];
    }
  };

  float kf[8], vf[8];
  int idx = k0 + wid * NR + sub;
#pragma unroll
  for (int j = 0; j < 8; ++j) kf[j] = vf[j] = 0.f;
  if (idx < k1) fetch(idx, kf, vf);
  for (int b = k0 + wid * NR; b < k1; b += 4 * NR, idx += 4 * NR) {
    float kx[8], vx[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) kx[j] = vx[j] = 0.f;
    if (idx + 4 * NR < k1) fetch(idx + 4 * NR, kx, vx);
    absorb(kf, vf, idx < k1);
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      kf[j] = kx[j];
      vf[j] = vx[j];
    }
  }
  if (a.append && split == 0 && wid == 0) {
    load8<VEC>(kn + d0, nd, kf);
    load8<VEC>(vn + d0, ne, vf);
    absorb(kf, vf, sub == 0);
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
      for (int j = 0; j < 8; ++j)
        o[r][j] = o[r][j] * c1 + __shfl_xor(o[r][j], off, 64) * c2;
    }
  __shared__ float so[4][RC][DV];
  __shared__ float sml[4][RC][2];
  if (sub == 0) {
#pragma unroll
    for (int r = 0; r < RC; ++r) {
#pragma unroll
      for (int j = 0; j < 8; ++j) so[wid][r][d0 + j] = o[r][j];
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

template <typename T>
__global__ void __launch_bounds__(64)
attn_rows_merge_kernel(const float* __restrict__ part, T* __restrict__ out,
                       int splits, int E) {
  const long rh = blockIdx.x;
  const float* p = part + rh * splits * (E + 2);
  float mm = NEG_BIG;
  for (int s = 0; s < splits; ++s) mm = fmaxf(mm, p[s * (E + 2) + E]);
  float ll = 0.f;
  for (int s = 0; s < splits; ++s)
    ll += p[s * (E + 2) + E + 1] *
          __builtin_amdgcn_exp2f(p[s * (E + 2) + E] - mm);
  const float inv = 1.f / ll;
  for (int e = threadIdx.x; e < E; e += 64) {
    float acc = 0.f;
    for (int s = 0; s < splits; ++s)
      acc += p[s * (E + 2) + e] *
             __builtin_amdgcn_exp2f(p[s * (E + 2) + E] - mm);
    from_f(out[rh * E + e], acc * inv);
  }
}

template <typename T>
static int launch_rows(const RowsArgs& a, int vec, hipStream_t stream) {
  const int rep = a.H / a.G;
  const int big = a.D > a.E ? a.D : a.E;
  const int rcn = rep >= 8 ? 8 : rep > 2 ? 4 : rep;
  const int nrc = (rep + rcn - 1) / rcn;
  const long grid = (long)a.rows * a.G * nrc * a.splits;
#define AR(L, R, V) attn_rows_kernel<T, L, R, V><<<grid, 256, 0, stream>>>(a)
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
  else return 1;
#undef ARR
#undef ARV
#undef AR
  if (a.splits > 1)
    attn_rows_merge_kernel<T><<<(long)a.rows * a.H, 64, 0, stream>>>(
        a.part, (T*)a.out, a.splits, a.E);
  return (int)hipGetLastError();
}

extern "C" int sv_attn_rows(const RowsArgs* a, int vec, int f32,
                            hipStream_t stream) {
  if (a->rows <= 0) return 0;
  return f32 ? launch_rows<float>(*a, vec, stream)
             : launch_rows<short>(*a, vec, stream);
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
// contraction order of P V, and V^T is read from LDS in the same order.
// ---------------------------------------------------------------------------
struct TilesArgs {
  const short* q;
  long qst;                 // row stride of q
  const short *kc, *vc;
  const int* tiles;         // [n_tiles][4]: seq, first row, rows, position
  const int* bt;
  short* out;               // [T][H * E]
  int MB, H, G, D, E, window, keep;
  float scale;
};

template <int DP, int NP>
__global__ void __launch_bounds__(256, DP <= 128 ? 2 : 1)
attn_tiles_kernel(TilesArgs a) {
  constexpr int NC = DP / 16;        // 16-wide chunks of the head size
  constexpr int NB = DP / 32;        // 32-row blocks of O^T
  constexpr int KP = DP * 2;         // K row pitch (bytes)
  constexpr int CPR = DP / 8;        // 16-byte slots of a row
  constexpr int PAIRS = 32 * CPR / 256;  // (row pair, slot) items a thread
  __shared__ __attribute__((aligned(16))) char kbuf[64 * KP];
  __shared__ __attribute__((aligned(16))) short vbuf[DP * 64];  // V^T

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
  const float s2 = a.scale * SV_LOG2E;

  const int q_hi = p0 + nrow - 1;
  const int t_hi = q_hi / SV_PAGE;
  const int lo = a.window > 0 ? max(0, p0 - a.window + 1) : 0;
  const int nk = a.window > 0
                     ? min((a.keep + SV_PAGE - 1) / SV_PAGE, t_hi + 1) : 0;
  const int t_lo = max(nk, lo / SV_PAGE);
  const int ntiles = nk + max(0, t_hi - t_lo + 1);
  const int w_lo = p0 + wid * 32, w_hi = min(w_lo + 31, q_hi);

  uint4v kreg[2 * PAIRS], vreg[2 * PAIRS];
  auto tile_of = [&](int n) { return n < nk ? n : t_lo + n - nk; };
  auto issue = [&](int n) {
    const long base = ((long)bt[tile_of(n)] * a.G + g) * SV_PAGE;
#pragma unroll
    for (int p = 0; p < PAIRS; ++p) {
      const int it = p * 256 + tid;
      const int r = it / CPR * 2, c = it % CPR * 8;
#pragma unroll
      for (int x = 0; x < 2; ++x) {
        kreg[2 * p + x] = c < D
            ? *(const uint4v*)(a.kc + (base + r + x) * D + c)
            : uint4v{0, 0, 0, 0};
        vreg[2 * p + x] = c < E
            ? *(const uint4v*)(a.vc + (base + r + x) * E + c)
            : uint4v{0, 0, 0, 0};
      }
    }
  };
  auto kswz = [](int row, int byte) {
    return CPR >= 16 ? swz16(row, byte) : swz(row, byte);
  };
  auto commit = [&]() {
#pragma unroll
    for (int p = 0; p < PAIRS; ++p) {
      const int it = p * 256 + tid;
      const int r = it / CPR * 2, c = it % CPR * 8;
      *(uint4v*)(kbuf + r * KP + kswz(r, c * 2)) = kreg[2 * p];
      *(uint4v*)(kbuf + (r + 1) * KP + kswz(r + 1, c * 2)) = kreg[2 * p + 1];
      union { uint4v u; unsigned short s[8]; } x, y;
      x.u = vreg[2 * p];
      y.u = vreg[2 * p + 1];
      const TileWrite tw(c, r);
#pragma unroll
      for (int j = 0; j < 8; ++j)
        *(uint*)(vbuf + tw.at(j)) = (uint)x.s[j] | ((uint)y.s[j] << 16);
    }
  };

  const TileRead vt(col, 4 * hi);
  issue(0);
  for (int n = 0; n < ntiles; ++n) {
    __syncthreads();           // readers of the previous tile are done
    commit();
    __syncthreads();
    if (n + 1 < ntiles) issue(n + 1);

    const int kv0 = tile_of(n) * SV_PAGE;
    const bool active = wid * 32 < nrow && kv0 <= w_hi &&
        (a.window <= 0 || kv0 < a.keep || kv0 + SV_PAGE - 1 > w_lo - a.window);
    if (!active) continue;

    f32x16 acc[2] = {};
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) {
      const int row = col + 32 * kb;
#pragma unroll
      for (int c = 0; c < NC; ++c) {
        frag_u kf;
        kf.u4 = *(const uint4v*)(kbuf + row * KP +
                                 kswz(row, (c * 16 + hi * 8) * 2));
        acc[kb] = mfma_bf16(kf.bf, qf[c].bf, acc[kb]);
      }
    }

    const bool masked = kv0 + SV_PAGE - 1 > w_lo ||
        (a.window > 0 && w_hi - kv0 >= a.window &&
         kv0 + SV_PAGE > a.keep);
    float mt = NEG_BIG;
#pragma unroll
    for (int kb = 0; kb < 2; ++kb)
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        float s = acc[kb][r] * s2;
        if (masked) {
          const int j = kv0 + 32 * kb + acc_row(r, hi);
          if (j > my_pos ||
              (a.window > 0 && my_pos - j >= a.window && j >= a.keep))
            s = NEG_BIG;
        }
        acc[kb][r] = s;
        mt = fmaxf(mt, s);
      }
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
        const int slot = 4 * kb + 2 * cc;
#pragma unroll
        for (int nb = 0; nb < NB; ++nb) {
          frag_u vf;
          *(uint2*)&vf.u[0] = *(const uint2*)(vbuf + vt.at(nb, slot));
          *(uint2*)&vf.u[2] = *(const uint2*)(vbuf + vt.at(nb, slot + 1));
#pragma unroll
          for (int z = 0; z < NP; ++z)
            ot[nb] = mfma_bf16(vf.bf, pf[z].bf, ot[nb]);
        }
      }
  }

  if (my >= nrow) return;
  const float inv = 1.f / l_run;
  short* dst = a.out + ((long)(row0 + my) * a.H + h) * E;
#pragma unroll
  for (int nb = 0; nb < NB; ++nb)
#pragma unroll
    for (int rg = 0; rg < 4; ++rg) {
      const int d = 32 * nb + 8 * rg + 4 * hi;
      if (d < E) {
        uint2 w = {pack_bf16x2(ot[nb][4 * rg] * inv, ot[nb][4 * rg + 1] * inv),
                   pack_bf16x2(ot[nb][4 * rg + 2] * inv,
                               ot[nb][4 * rg + 3] * inv)};
        *(uint2*)(dst + d) = w;
      }
    }
}

// D and E multiples of 8, at most 256; q rows 16-byte aligned
extern "C" int sv_attn_tiles(const TilesArgs* a, int n_tiles,
                             hipStream_t stream) {
  if (n_tiles <= 0) return 0;
  const int big = a->D > a->E ? a->D : a->E;
  const dim3 grid(a->H, n_tiles);
  if (big <= 64) attn_tiles_kernel<64, 3><<<grid, 256, 0, stream>>>(*a);
  else if (big <= 128) attn_tiles_kernel<128, 3><<<grid, 256, 0, stream>>>(*a);
  else if (big <= 256) attn_tiles_kernel<256, 3><<<grid, 256, 0, stream>>>(*a);
  else return 1;
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
