// Element access shared by the row, attention and recurrence kernels.
#pragma once
#include "socket_common.h"

template <class DT>
__device__ __forceinline__ float load_elem(const void* p, int64_t i);
template <>
__device__ __forceinline__ float load_elem<DType_f32>(const void* p, int64_t i) { return ((const float*)p)[i]; }
template <>
__device__ __forceinline__ float load_elem<DType_bf16>(const void* p, int64_t i) {
  return bf16_bits_to_f32(((const uint16_t*)p)[i]);
}

// N consecutive elements (N = 1, 4 or 8) as floats; for N > 1 the address must be aligned to
// N elements of the type (16 bytes at most).
template <class DT, int N>
__device__ __forceinline__ void load_vec(const void* p, int64_t i, float* out) {
  if constexpr (N == 1) {
    out[0] = load_elem<DT>(p, i);
  } else if constexpr (DT::kPer16B == 4) {
#pragma unroll
    for (int k = 0; k < N; k += 4)
      unpack16<DT>(*reinterpret_cast<const uint4*>((const float*)p + i + k), out + k);
  } else if constexpr (N == 8) {
    unpack16<DT>(*reinterpret_cast<const uint4*>((const uint16_t*)p + i), out);
  } else {
    const uint2 w = *reinterpret_cast<const uint2*>((const uint16_t*)p + i);
    out[0] = __uint_as_float(w.x << 16);
    out[1] = __uint_as_float(w.x & 0xffff0000u);
    out[2] = __uint_as_float(w.y << 16);
    out[3] = __uint_as_float(w.y & 0xffff0000u);
  }
}

template <class DT, int N>
__device__ __forceinline__ void store_vec(void* p, int64_t i, const float* v) {
  if constexpr (N == 1) {
    store_elem<DT>(p, i, v[0]);
  } else if constexpr (DT::kPer16B == 4) {
#pragma unroll
    for (int k = 0; k < N; k += 4)
      *reinterpret_cast<float4*>((float*)p + i + k) = make_float4(v[k], v[k + 1], v[k + 2], v[k + 3]);
  } else {
    uint32_t w[N / 2];
#pragma unroll
    for (int k = 0; k < N / 2; ++k)
      w[k] = (uint32_t)f32_to_bf16_bits(v[2 * k]) | ((uint32_t)f32_to_bf16_bits(v[2 * k + 1]) << 16);
    if constexpr (N == 8) *reinterpret_cast<uint4*>((uint16_t*)p + i) = make_uint4(w[0], w[1], w[2], w[3]);
    else *reinterpret_cast<uint2*>((uint16_t*)p + i) = make_uint2(w[0], w[1]);
  }
}

// The hardware's base-2 exponential and logarithm, reciprocal and reciprocal square root, each
// accurate to about one unit in the last place, instead of the math library's versions: the
// kernels of a decode step run once per token with cold instruction caches, where every
// line of code is a trip to memory.
constexpr float kElemLog2e = 1.4426950408889634f, kElemLn2 = 0.6931471805599453f;
__device__ __forceinline__ float exp_f32(float x) { return __builtin_amdgcn_exp2f(x * kElemLog2e); }
__device__ __forceinline__ float rsqrt_f32(float x) { return __builtin_amdgcn_rsqf(x); }
__device__ __forceinline__ float sigmoid_f32(float x) { return __builtin_amdgcn_rcpf(1.f + exp_f32(-x)); }
// log(1 + t) for t >= 0 without losing what rounding 1 + t drops: log(u) * t / (u - 1) with u the
// rounded 1 + t (W. Kahan's method; D. Goldberg, "What Every Computer Scientist Should Know About
// Floating-Point Arithmetic", 1991).
__device__ __forceinline__ float log1p_f32(float t) {
  const float u = 1.f + t, d = u - 1.f;
  return d == 0.f ? t : __builtin_amdgcn_logf(u) * kElemLn2 * (t * __builtin_amdgcn_rcpf(d));
}
__device__ __forceinline__ float softplus_f32(float x) { return fmaxf(x, 0.f) + log1p_f32(exp_f32(-fabsf(x))); }

// 1 - 2 / (e^2x + 1): exact to about one unit of the result's scale 1 (the argument's own scale
// near 0, where the difference cancels, is served by the odd polynomial's first terms).
__device__ __forceinline__ float tanh_f32(float x) {
  const float big = 1.f - 2.f * __builtin_amdgcn_rcpf(exp_f32(2.f * x) + 1.f);
  const float x2 = x * x;
  const float small = x * fmaf(x2, fmaf(x2, 2.f / 15.f, -1.f / 3.f), 1.f);
  return fabsf(x) < 0.05f ? small : big;
}

// Sum over the workgroup (a multiple of 64 lanes, up to 1024), the same value in every lane.
// `red` holds one float per wave; two calls in a row need two arrays or a barrier between.
__device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_reduce_to_last<false>(v);
  if ((threadIdx.x & 63) == 63) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float tot = 0.f;
  for (int k = 0; k < (int)(blockDim.x >> 6); ++k) tot += red[k];
  return tot;
}
