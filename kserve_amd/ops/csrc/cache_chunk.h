// Pieces of paged-cache rows in registers, shared by the attention kernels that
// compute in fp32 over bf16 or fp32 pages.
#pragma once

#include "dtype_io.h"

typedef float f32x4 __attribute__((ext_vector_type(4)));

// 8 consecutive elements of a cache row, kept in the cache dtype while the
// load is in flight (a bf16 chunk costs 4 registers) and widened on the way
// into LDS
template <typename T>
struct Chunk8;
template <>
struct Chunk8<short> {
  short8_t x;
  __device__ __forceinline__ void load(const short* p, bool vec, int valid) {
    if (vec && valid >= 8) {
      x = *reinterpret_cast<const short8_t*>(p);
    } else {
#pragma unroll
      for (int i = 0; i < 8; ++i) x[i] = i < valid ? p[i] : (short)0;
    }
  }
  __device__ __forceinline__ void zero() {
#pragma unroll
    for (int i = 0; i < 8; ++i) x[i] = 0;
  }
  __device__ __forceinline__ float get(int i) const { return bf16_bits_to_float(x[i]); }
};
template <>
struct Chunk8<float> {
  f32x4 a, b;
  __device__ __forceinline__ void load(const float* p, bool vec, int valid) {
    if (vec && valid >= 8) {
      a = *reinterpret_cast<const f32x4*>(p);
      b = *reinterpret_cast<const f32x4*>(p + 4);
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        a[i] = i < valid ? p[i] : 0.f;
        b[i] = 4 + i < valid ? p[4 + i] : 0.f;
      }
    }
  }
  __device__ __forceinline__ void zero() {
    a = f32x4{0.f, 0.f, 0.f, 0.f};
    b = a;
  }
  __device__ __forceinline__ float get(int i) const { return i < 4 ? a[i] : b[i - 4]; }
};

// four consecutive elements as fp32, the last `valid` < 4 of a row guarded;
// `vec`: rows and columns are 4-element aligned
template <typename T>
__device__ __forceinline__ f32x4 load4_f32(const T* p, bool vec, int valid);
template <>
__device__ __forceinline__ f32x4 load4_f32<short>(const short* p, bool vec,
                                                  int valid) {
  f32x4 r = f32x4{0.f, 0.f, 0.f, 0.f};
  if (vec && valid >= 4) {
    const short4_t x = *reinterpret_cast<const short4_t*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) r[i] = bf16_bits_to_float(x[i]);
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (i < valid) r[i] = bf16_bits_to_float(p[i]);
  }
  return r;
}
template <>
__device__ __forceinline__ f32x4 load4_f32<float>(const float* p, bool vec,
                                                  int valid) {
  f32x4 r = f32x4{0.f, 0.f, 0.f, 0.f};
  if (vec && valid >= 4) {
    r = *reinterpret_cast<const f32x4*>(p);
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (i < valid) r[i] = p[i];
  }
  return r;
}
