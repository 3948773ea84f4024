// Fragments of 16 x 16 products over 32 k's for kernels served in bf16 and in fp32.  Lane (m = lane & 15, g = lane >> 4) holds
// k = 8 g .. 8 g + 7 of row (A) or column (B) m; a result lane holds rows 4 g .. 4 g + 3 of column m.
//
// Frag<T>: eight elements as stored.  Wide<T>: eight fp32 values; in the bf16 build three bf16 terms (8 + 8 + 8 significant bits)
// that are multiplied one after another, so a product of a Wide with a Frag is exact up to the fp32 sums.  In the fp32 build both are
// floats and a product is eight v_mfma_f32_16x16x4_f32, whose k-slot g of product i stands for k = 8 g + i.
#pragma once
#include "hybrid.h"

namespace {

template <typename T> struct Frag;
template <typename T> struct Wide;
template <> struct Frag<bf16_t> { uint4 v; };
template <> struct Frag<float> { float v[8]; };
template <> struct Wide<bf16_t> { uint4 t[3]; };
template <> struct Wide<float> { float v[8]; };

__device__ __forceinline__ void frag_load(Frag<bf16_t>& f, const bf16_t* p) { f.v = *reinterpret_cast<const uint4*>(p); }
__device__ __forceinline__ void frag_load(Frag<float>& f, const float* p) {
  const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
  f.v[0] = a.x; f.v[1] = a.y; f.v[2] = a.z; f.v[3] = a.w; f.v[4] = b.x; f.v[5] = b.y; f.v[6] = b.z; f.v[7] = b.w;
}
__device__ __forceinline__ void frag_zero(Frag<bf16_t>& f) { f.v = make_uint4(0, 0, 0, 0); }
__device__ __forceinline__ void frag_zero(Frag<float>& f) {
#pragma unroll
  for (int i = 0; i < 8; ++i) f.v[i] = 0.f;
}

// two fp32 values as three packed bf16 pairs whose sum is exact
__device__ __forceinline__ void split_pair(float a, float b, uint32_t& hi, uint32_t& mid, uint32_t& lo) {
  hi = pack_bf(a, b);
  const float r0 = a - lo_bf(hi), r1 = b - hi_bf(hi);
  mid = pack_bf(r0, r1);
  lo = pack_bf(r0 - lo_bf(mid), r1 - hi_bf(mid));
}
__device__ __forceinline__ void wide_from(Wide<bf16_t>& w, const float* v) {
  uint32_t h[4], m[4], l[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) split_pair(v[2 * e], v[2 * e + 1], h[e], m[e], l[e]);
  w.t[0] = make_uint4(h[0], h[1], h[2], h[3]);
  w.t[1] = make_uint4(m[0], m[1], m[2], m[3]);
  w.t[2] = make_uint4(l[0], l[1], l[2], l[3]);
}
__device__ __forceinline__ void wide_from(Wide<float>& w, const float* v) {
#pragma unroll
  for (int i = 0; i < 8; ++i) w.v[i] = v[i];
}

// A matrix of fp32 values in LDS that is read as Wide fragments: three planes of bf16, or floats.  `plane`: elements of one.
template <typename T> struct WideLds;
template <> struct WideLds<bf16_t> {
  static constexpr int PLANES = 3;
  static __device__ __forceinline__ void put4(bf16_t* p, int plane, const float* v) {
    uint32_t h[2], m[2], l[2];
#pragma unroll
    for (int e = 0; e < 2; ++e) split_pair(v[2 * e], v[2 * e + 1], h[e], m[e], l[e]);
    *reinterpret_cast<uint2*>(p) = make_uint2(h[0], h[1]);
    *reinterpret_cast<uint2*>(p + plane) = make_uint2(m[0], m[1]);
    *reinterpret_cast<uint2*>(p + 2 * plane) = make_uint2(l[0], l[1]);
  }
  static __device__ __forceinline__ void get(Wide<bf16_t>& w, const bf16_t* p, int plane) {
#pragma unroll
    for (int i = 0; i < 3; ++i) w.t[i] = *reinterpret_cast<const uint4*>(p + i * plane);
  }
};
template <> struct WideLds<float> {
  static constexpr int PLANES = 1;
  static __device__ __forceinline__ void put4(float* p, int, const float* v) {
    *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
  }
  static __device__ __forceinline__ void get(Wide<float>& w, const float* p, int) {
    const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
    w.v[0] = a.x; w.v[1] = a.y; w.v[2] = a.z; w.v[3] = a.w; w.v[4] = b.x; w.v[5] = b.y; w.v[6] = b.z; w.v[7] = b.w;
  }
};

__device__ __forceinline__ f32x4 mma_bf(uint4 a, uint4 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}
__device__ __forceinline__ f32x4 mma_f(const float* a, const float* b, f32x4 c) {
#pragma unroll
  for (int i = 0; i < 8; ++i) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[i], c, 0, 0, 0);
  return c;
}
__device__ __forceinline__ f32x4 mma(const Frag<bf16_t>& a, const Frag<bf16_t>& b, f32x4 c) { return mma_bf(a.v, b.v, c); }
__device__ __forceinline__ f32x4 mma(const Wide<bf16_t>& a, const Frag<bf16_t>& b, f32x4 c) {
#pragma unroll
  for (int i = 0; i < 3; ++i) c = mma_bf(a.t[i], b.v, c);
  return c;
}
__device__ __forceinline__ f32x4 mma(const Frag<bf16_t>& a, const Wide<bf16_t>& b, f32x4 c) {
#pragma unroll
  for (int i = 0; i < 3; ++i) c = mma_bf(a.v, b.t[i], c);
  return c;
}
__device__ __forceinline__ f32x4 mma(const Frag<float>& a, const Frag<float>& b, f32x4 c) { return mma_f(a.v, b.v, c); }
__device__ __forceinline__ f32x4 mma(const Wide<float>& a, const Frag<float>& b, f32x4 c) { return mma_f(a.v, b.v, c); }
__device__ __forceinline__ f32x4 mma(const Frag<float>& a, const Wide<float>& b, f32x4 c) { return mma_f(a.v, b.v, c); }

}  // namespace
