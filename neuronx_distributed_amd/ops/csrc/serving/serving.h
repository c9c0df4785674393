// Shared helpers of the serving kernels (ragged batches, 32-bit residual).
//
// Every kernel here is written for an element type T of activations and
// weights: `short` holds bf16 bits, `float` is the true 32-bit mode.
#pragma once

#include "../common.h"
#include "../mfma.h"

#define SV_PAGE 64  // tokens of one cache page
#define SV_LOG2E 1.4426950408889634f

typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef short s4v __attribute__((ext_vector_type(4)));

// operands of direct loads into LDS and of transposing LDS loads
typedef __attribute__((address_space(1))) const void* global_ptr;
typedef __attribute__((address_space(3))) void* lds_ptr;
typedef short tr4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) tr4* lds_tr4;

__device__ __forceinline__ float to_f(short v) { return bits2f(v); }
__device__ __forceinline__ float to_f(float v) { return v; }
__device__ __forceinline__ void from_f(short& o, float v) { o = f2bits(v); }
__device__ __forceinline__ void from_f(float& o, float v) { o = v; }

// 4 elements at p[0..3] (16 B / 8 B aligned)
__device__ __forceinline__ void load4(const float* p, float* v) {
  const f32x4 a = *(const f32x4*)p;
#pragma unroll
  for (int j = 0; j < 4; ++j) v[j] = a[j];
}
__device__ __forceinline__ void load4(const short* p, float* v) {
  const s4v a = *(const s4v*)p;
#pragma unroll
  for (int j = 0; j < 4; ++j) v[j] = bits2f(a[j]);
}
__device__ __forceinline__ void store4(float* p, const float* v) {
  f32x4 a;
#pragma unroll
  for (int j = 0; j < 4; ++j) a[j] = v[j];
  *(f32x4*)p = a;
}
__device__ __forceinline__ void store4(short* p, const float* v) {
  s4v a;
#pragma unroll
  for (int j = 0; j < 4; ++j) a[j] = f2bits(v[j]);
  *(s4v*)p = a;
}

// 8 elements; `n` of them are inside the row, the rest read as zero.  VEC
// promises 8-element alignment and a row length that is a multiple of 8.
template <bool VEC, typename T>
__device__ __forceinline__ void load8(const T* p, int n, float* v) {
  if (VEC) {
    if (n > 0) {
      load4(p, v);
      load4(p + 4, v + 4);
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] = 0.f;
    }
  } else {
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = j < n ? to_f(p[j]) : 0.f;
  }
}

template <>
__device__ __forceinline__ void load8<true, short>(const short* p, int n,
                                                   float* v) {
  const s8v a = n > 0 ? *(const s8v*)p : s8v{0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
  for (int j = 0; j < 8; ++j) v[j] = bits2f(a[j]);
}

// v_rcp_f32 and v_exp_f32 are good to one unit in the last place
__device__ __forceinline__ float sigmoid_f(float x) {
  return __builtin_amdgcn_rcpf(1.f +
                               __builtin_amdgcn_exp2f(-x * SV_LOG2E));
}
__device__ __forceinline__ float silu_f(float x) { return x * sigmoid_f(x); }
// log(sigmoid(x)), stable on both sides
__device__ __forceinline__ float log_sigmoid_f(float x) {
  return fminf(x, 0.f) - log1pf(expf(-fabsf(x)));
}

// cos and sin of position p of a pair that turns f radians a position.  The
// angle is reduced in double, so its error does not grow with the
// position.
__device__ __forceinline__ void turn(double f, int p, float* c, float* s) {
  const double a = f * p;
  const double r = a - rint(a * 0.15915494309189535) * 6.283185307179586;
  sincosf((float)r, s, c);
}

// s-contiguous tile [rows][64] without padding: 16-byte slots are rotated so
// that both the pairwise transposing writes (fixed row low bits) and the
// fragment reads (consecutive rows) spread over the banks
__device__ __forceinline__ int tslot(int row, int s) {
  return row * 64 + ((((s >> 3) ^ (row >> 1) ^ (row >> 4)) & 7) << 3) +
         (s & 7);
}

// Lane part of the tile's addresses, so that an access costs one xor and an
// immediate offset.
struct TileRead {            // row = 32 nb + col, s = 8 slot + 4 hi (+ 0..7)
  int base;                  // elements, slot bits xor-ed in later
  __device__ __forceinline__ TileRead(int col, int low)
      : base(col * 64 + ((((col >> 1) ^ (col >> 4)) & 7) << 3) + low) {}
  __device__ __forceinline__ int at(int nb, int slot) const {
    return (base ^ (((slot ^ (2 * nb)) & 7) << 3)) + nb * 2048;
  }
};
struct TileWrite {           // row = c + j (c a multiple of 8), s = r
  int base;
  __device__ __forceinline__ TileWrite(int c, int r)
      : base(c * 64 + ((((r >> 3) ^ ((c >> 1) & 4) ^ (c >> 4)) & 7) << 3) +
             (r & 7)) {}
  __device__ __forceinline__ int at(int j) const {
    return (base ^ ((j >> 1) << 3)) + j * 64;
  }
};
