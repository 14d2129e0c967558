// Eight consecutive elements of a bf16 or fp32 row to and from fp32 registers, and the layouts
// the head kernels (qkv_heads.hip, conv_heads.hip) share.
#pragma once
#include "common.h"
#include "kernels.h"

namespace oamd {

template <typename T>
__device__ __forceinline__ void st8(T* p, const float (&v)[8]);
template <>
__device__ __forceinline__ void st8<float>(float* p, const float (&v)[8]) {
  *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
  *reinterpret_cast<f32x4*>(p + 4) = f32x4{v[4], v[5], v[6], v[7]};
}
template <>
__device__ __forceinline__ void st8<bf16_t>(bf16_t* p, const float (&v)[8]) {
  *reinterpret_cast<uint4*>(p) =
      make_uint4(pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3]), pack_bf2(v[4], v[5]), pack_bf2(v[6], v[7]));
}

template <typename T>
__device__ __forceinline__ void ld8(const T* p, float (&v)[8]);
template <>
__device__ __forceinline__ void ld8<float>(const float* p, float (&v)[8]) {
  const f32x4 a = *reinterpret_cast<const f32x4*>(p), b = *reinterpret_cast<const f32x4*>(p + 4);
#pragma unroll
  for (int j = 0; j < 4; ++j) v[j] = a[j], v[4 + j] = b[j];
}
template <>
__device__ __forceinline__ void ld8<bf16_t>(const bf16_t* p, float (&v)[8]) {
  const u16x8 a = *reinterpret_cast<const u16x8*>(p);
#pragma unroll
  for (int j = 0; j < 8; ++j) v[j] = bf2f(a[j]);
}

// eight elements kept as they are stored
template <typename T>
struct Raw8;
template <>
struct Raw8<float> {
  float v[8];
};
template <>
struct Raw8<bf16_t> {
  u16x8 v;
};
__device__ __forceinline__ float raw_at(const Raw8<float>& r, int j) { return r.v[j]; }
__device__ __forceinline__ float raw_at(const Raw8<bf16_t>& r, int j) { return bf2f(r.v[j]); }
template <typename T>
__device__ __forceinline__ Raw8<T> raw_zero() {
  Raw8<T> r;
#pragma unroll
  for (int j = 0; j < 8; ++j) r.v[j] = 0;
  return r;
}
template <typename T>
__device__ __forceinline__ Raw8<T> raw_ld(const T* p) {
  Raw8<T> r;
  if constexpr (sizeof(T) == 4) ld8<float>(p, r.v);
  else r.v = *reinterpret_cast<const u16x8*>(p);
  return r;
}
template <typename T>
__device__ __forceinline__ void raw_st(T* p, const Raw8<T>& r) {
  if constexpr (sizeof(T) == 4) st8<float>(p, r.v);
  else *reinterpret_cast<u16x8*>(p) = r.v;
}

// columns col..col+7 of row t of a projection: rows [T][ncol], or the sum of S fp32 slabs
template <typename T>
__device__ __forceinline__ void load_row8(const float* xp, const void* row, int S, int64_t slab, int64_t at, float (&v)[8]) {
  if (xp) {
    float w[8][8];   // up to 8 slabs requested before the first add
#pragma unroll
    for (int s = 0; s < 8; ++s)
      if (s < S) ld8<float>(xp + at + s * slab, w[s]);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = w[0][j];
#pragma unroll
    for (int s = 1; s < 8; ++s)
      if (s < S) {
#pragma unroll
        for (int j = 0; j < 8; ++j) v[j] += w[s][j];
      }
    for (int s = 8; s < S; ++s) {
      ld8<float>(xp + at + s * slab, w[0]);
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] += w[0][j];
    }
  } else {
    ld8<T>(static_cast<const T*>(row) + at, v);
  }
}

// the same in the row type (slabs are summed, then rounded)
template <typename T>
__device__ __forceinline__ Raw8<T> raw_row8(const float* xp, const void* row, int S, int64_t slab, int64_t at) {
  if (!xp) return raw_ld<T>(static_cast<const T*>(row) + at);
  float v[8];
  load_row8<T>(xp, row, S, slab, at, v);
  Raw8<T> r;
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    if constexpr (sizeof(T) == 4) r.v[j] = v[j];
    else r.v[j] = f2bf(v[j]);
  }
  return r;
}

// one element of the same
template <typename T>
__device__ __forceinline__ float load_row1(const float* xp, const void* row, int S, int64_t slab, int64_t at) {
  if (xp) {
    float w[8];
#pragma unroll
    for (int s = 0; s < 8; ++s) w[s] = s < S ? xp[at + s * slab] : 0.f;
    float v = w[0];
#pragma unroll
    for (int s = 1; s < 8; ++s) v += w[s];
    for (int s = 8; s < S; ++s) v += xp[at + s * slab];
    return v;
  }
  if constexpr (sizeof(T) == 4) return static_cast<const float*>(row)[at];
  else return bf2f(static_cast<const bf16_t*>(row)[at]);
}

template <typename T>
__device__ __forceinline__ void st1(T* p, float v) {
  if constexpr (sizeof(T) == 4) *p = v;
  else *p = f2bf(v);
}

// Cache writes of 8 dims (chunk c) of a key / value head whose page starts at row `head` (page * Hkv +
// kv head) << log2_page, token `off` of the page: fp32 token rows, or the bf16 tiles the decode
// attention reads as MFMA fragments (K [d / 8][16 token][8 dims]; V [d / 32][4 token group][16 dims][2 half][4 token]).
template <typename T>
__device__ __forceinline__ void cache_k8(T* dst, int64_t head, int off, int dkp, int c, const float (&x)[8]) {
  if constexpr (sizeof(T) == 4) dst += (head + off) * dkp + 8 * c;
  else dst += (head + (off & ~15)) * dkp + (c * 16 + (off & 15)) * 8;
  st8<T>(dst, x);
}
template <typename T>
__device__ __forceinline__ void cache_v8(T* dst, int64_t head, int off, int dvp, int c, const float (&x)[8]) {
  if constexpr (sizeof(T) == 4) {
    st8<T>(dst + (head + off) * dvp + 8 * c, x);
  } else {
    const int d0 = 8 * c, t16 = off & 15;
    dst += (head + (off & ~15)) * dvp + (((d0 >> 5) * 4 + (t16 >> 2)) * 16 + (d0 & 15)) * 8 + ((d0 >> 4) & 1) * 4 + (t16 & 3);
#pragma unroll
    for (int j = 0; j < 8; ++j) dst[8 * j] = f2bf(x[j]);
  }
}

}  // namespace oamd
