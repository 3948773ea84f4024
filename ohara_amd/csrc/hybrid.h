// Shared by the kernels of hybrid decoders (residual_norm.hip, attention_bias.hip, delta_rule.hip): typed
// loads and stores (bf16 or fp32 activations) and the row bookkeeping of OharaSeq.
#pragma once
#include "common.h"

namespace {

__device__ __forceinline__ float ldv(const bf16_t* p) { return bf2f(*p); }
__device__ __forceinline__ float ldv(const float* p) { return *p; }
__device__ __forceinline__ void stv(bf16_t* p, float v) { *p = f2bf(v); }
__device__ __forceinline__ void stv(float* p, float v) { *p = v; }

// four / eight consecutive elements (the pointer is aligned to the piece)
__device__ __forceinline__ void ld4(const bf16_t* p, float* o) {
  const uint2 v = ldg8(p);
  o[0] = lo_bf(v.x); o[1] = hi_bf(v.x); o[2] = lo_bf(v.y); o[3] = hi_bf(v.y);
}
__device__ __forceinline__ void ld4(const float* p, float* o) {
  const uint4 v = ldg16(p);
  o[0] = __uint_as_float(v.x); o[1] = __uint_as_float(v.y); o[2] = __uint_as_float(v.z); o[3] = __uint_as_float(v.w);
}
__device__ __forceinline__ void st4(bf16_t* p, const float* v) { stg8(p, make_uint2(pack_bf(v[0], v[1]), pack_bf(v[2], v[3]))); }
__device__ __forceinline__ void st4(float* p, const float* v) {
  *(OHARA_GLOBAL u32x4*)p = (u32x4){__float_as_uint(v[0]), __float_as_uint(v[1]), __float_as_uint(v[2]), __float_as_uint(v[3])};
}

// eight elements as loaded (registers), unpacked when they are used
template <typename T> struct Raw8;
template <> struct Raw8<bf16_t> {
  uint4 v;
  __device__ __forceinline__ void load(const bf16_t* p) { v = ldg16(p); }
  __device__ __forceinline__ void zero() { v = make_uint4(0, 0, 0, 0); }
  __device__ __forceinline__ void get(float* o) const {
    o[0] = lo_bf(v.x); o[1] = hi_bf(v.x); o[2] = lo_bf(v.y); o[3] = hi_bf(v.y);
    o[4] = lo_bf(v.z); o[5] = hi_bf(v.z); o[6] = lo_bf(v.w); o[7] = hi_bf(v.w);
  }
};
template <> struct Raw8<float> {
  uint4 a, b;
  __device__ __forceinline__ void load(const float* p) { a = ldg16(p); b = ldg16(p + 4); }
  __device__ __forceinline__ void zero() { a = b = make_uint4(0, 0, 0, 0); }
  __device__ __forceinline__ void get(float* o) const {
    o[0] = __uint_as_float(a.x); o[1] = __uint_as_float(a.y); o[2] = __uint_as_float(a.z); o[3] = __uint_as_float(a.w);
    o[4] = __uint_as_float(b.x); o[5] = __uint_as_float(b.y); o[6] = __uint_as_float(b.z); o[7] = __uint_as_float(b.w);
  }
};

__device__ __forceinline__ int seq_start(const OharaSeq& q, int b) {
  return q.pos_dev ? q.pos_dev[(size_t)b * q.pos_stride] : q.pos;
}
__device__ __forceinline__ int seq_tokens(const OharaSeq& q, int b) { return q.lens ? min(q.lens[b], q.seq_len) : q.seq_len; }
__device__ __forceinline__ int seq_slot(const OharaSeq& q, int b) { return q.slots ? q.slots[b] : b; }

// sigmoid, silu and softplus in fp32 on the hardware exponential, logarithm and reciprocal (each within a few units of the
// last place; the library functions and the IEEE division are several times the instructions)
__device__ __forceinline__ float sigmoid_x(float v) { return __frcp_rn(1.0f + __expf(-v)); }
__device__ __forceinline__ float silu_x(float v) { return v * __frcp_rn(1.0f + __expf(-v)); }
// max(v, 0) + log(1 + e) with e = exp(-|v|).  1 + e rounds; dividing by what it rounded to, log(u) * e / (u - 1) with
// u = fl(1 + e), keeps the relative precision for small e.
__device__ __forceinline__ float softplus_x(float v) {
  const float e = __expf(-fabsf(v)), u = 1.0f + e, d = u - 1.0f;
  const float l = d == 0.f ? e : __logf(u) * e * __frcp_rn(d);
  return fmaxf(v, 0.f) + l;
}

inline bool seq_ok(const OharaSeq* q) {
  return q && q->batch >= 1 && q->seq_len >= 1 && (int64_t)q->batch * q->seq_len <= INT32_MAX &&
         (q->pos_stride == 0 || q->pos_stride == 1) && (q->pos_dev || q->pos >= 0);
}

}  // namespace
