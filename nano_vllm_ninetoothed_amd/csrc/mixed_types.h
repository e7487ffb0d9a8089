// Loads and stores for kernels that exist in bfloat16 and in float: every value is a float in registers, the element
// type only decides what lies in memory.  VEC consecutive elements move as 16-byte pieces where the caller has checked
// that the addresses allow it (VEC = 8), else one by one (VEC = 1).
#pragma once
#include "mops_common.h"

namespace mops {

struct bf16_t { uint16_t bits; };

__device__ __forceinline__ float to_f32(float v) { return v; }
__device__ __forceinline__ float to_f32(bf16_t v) { return __uint_as_float((uint32_t)v.bits << 16); }
template <typename T> __device__ __forceinline__ T from_f32(float v);
template <> __device__ __forceinline__ float from_f32<float>(float v) { return v; }
template <> __device__ __forceinline__ bf16_t from_f32<bf16_t>(float v) { return bf16_t{(uint16_t)f32_to_bf16_bits(v)}; }

template <int VEC> __device__ __forceinline__ void load_vec(const float* p, float (&v)[VEC]) {
  if (VEC % 4 == 0) {
#pragma unroll
    for (int i = 0; i < VEC / 4; ++i) {
      const f32x4 w = *reinterpret_cast<const f32x4*>(p + 4 * i);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[(4 * i + e) % VEC] = w[e];
    }
  } else {
#pragma unroll
    for (int i = 0; i < VEC; ++i) v[i] = p[i];
  }
}
template <int VEC> __device__ __forceinline__ void load_vec(const bf16_t* p, float (&v)[VEC]) {
  if (VEC % 8 == 0) {
#pragma unroll
    for (int i = 0; i < VEC / 8; ++i) {
      const u32x4 w = load16(p + 8 * i);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        v[(8 * i + 2 * e) % VEC] = bf16lo_to_f32(w[e]);
        v[(8 * i + 2 * e + 1) % VEC] = bf16hi_to_f32(w[e]);
      }
    }
  } else {
#pragma unroll
    for (int i = 0; i < VEC; ++i) v[i] = to_f32(p[i]);
  }
}
template <int VEC> __device__ __forceinline__ void store_vec(float* p, const float (&v)[VEC]) {
  if (VEC % 4 == 0) {
#pragma unroll
    for (int i = 0; i < VEC / 4; ++i) {
      f32x4 w;
#pragma unroll
      for (int e = 0; e < 4; ++e) w[e] = v[(4 * i + e) % VEC];
      *reinterpret_cast<f32x4*>(p + 4 * i) = w;
    }
  } else {
#pragma unroll
    for (int i = 0; i < VEC; ++i) p[i] = v[i];
  }
}
template <int VEC> __device__ __forceinline__ void store_vec(bf16_t* p, const float (&v)[VEC]) {
  if (VEC % 8 == 0) {
#pragma unroll
    for (int i = 0; i < VEC / 8; ++i) {
      u32x4 w;
#pragma unroll
      for (int e = 0; e < 4; ++e) w[e] = pack_bf16x2(v[(8 * i + 2 * e) % VEC], v[(8 * i + 2 * e + 1) % VEC]);
      store16(p + 8 * i, w);
    }
  } else {
#pragma unroll
    for (int i = 0; i < VEC; ++i) p[i] = from_f32<bf16_t>(v[i]);
  }
}

// 1 / (1 + e^-v) for results of type T: bf16 from the hardware's base-2 exponential and reciprocal (about one ulp of float32
// each), float from the library's exponential and a true division.
template <typename T> __device__ __forceinline__ float sigmoid_for(float v) {
  return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * v));
}
template <> __device__ __forceinline__ float sigmoid_for<float>(float v) { return 1.0f / (1.0f + expf(-v)); }
template <typename T> __device__ __forceinline__ float silu_for(float v) { return v * sigmoid_for<T>(v); }
// log(1 + e^v); beyond 20 the difference to v is below one ulp of v.
__device__ __forceinline__ float softplus_f32(float v) { return v > 20.0f ? v : log1pf(expf(v)); }
// The same from the hardware's base-2 exponential and logarithm, a relative error of about 1e-6: where 1 + e^v would lose e^v's digits
// the logarithm is its series.
__device__ __forceinline__ float softplus_fast(float v) {
  const float y = __builtin_amdgcn_exp2f(1.4426950408889634f * v);
  const float series = y * (1.0f - y * (0.5f - y * (0.33333333f - 0.25f * y)));
  return v > 20.0f ? v : (y < 0.03125f ? series : 0.6931471805599453f * __builtin_amdgcn_logf(1.0f + y));
}

// Sum over the whole workgroup of THREADS threads; every thread gets the total.  Contains two barriers.
template <int THREADS>
__device__ __forceinline__ float block_sum(float v, float* scratch /* [THREADS / kWave] in LDS */) {
  v = group_sum<kWave>(v);
  if (THREADS <= kWave) return v;
  __syncthreads();
  if ((threadIdx.x & (kWave - 1)) == 0) scratch[threadIdx.x / kWave] = v;
  __syncthreads();
  float s = 0.f;
#pragma unroll
  for (int w = 0; w < THREADS / kWave; ++w) s += scratch[w];
  return s;
}

// Element types of the mixed-type entry points.
inline bool known_dtype(int dtype) { return dtype == MOPS_HIP_BF16 || dtype == MOPS_HIP_F32; }

}  // namespace mops
