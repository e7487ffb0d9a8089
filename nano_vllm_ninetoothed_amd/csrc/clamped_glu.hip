// Gated units over [rows, n]; gate and up are usually the two halves of one projection and are read in place.
//   clamped_glu    out = g * sigmoid(alpha * g) * (u + 1) with g = min(gate, limit), u = clamp(up, -limit, limit)
//   gelu_glu       out = gelu(gate) * up, gelu in its tanh form
//   relu_glu       out = max(gate, 0) * up
#include "mixed_types.h"

namespace mops {

// z (1 + tanh(c (z + 0.044715 z^3))) / 2 = z / (1 + e^(-2 c (z + 0.044715 z^3))), c = sqrt(2 / pi)
template <typename T> __device__ __forceinline__ float gelu_tanh(float z) {
  return z * sigmoid_for<T>(1.5957691216057308f * (z + 0.044715f * z * z * z));
}

enum GatedUnit { kClamped, kGelu, kRelu };

template <typename T, int VEC, GatedUnit UNIT>
__global__ __launch_bounds__(256) void clamped_glu_kernel(const T* __restrict__ gate, int64_t gate_stride, const T* __restrict__ up,
                                                          int64_t up_stride, T* __restrict__ out, int64_t out_stride, int64_t rows, int n,
                                                          float alpha, float limit) {
  const int pieces = n / VEC;
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= rows * pieces) return;
  const int64_t row = i / pieces;
  const int c = (int)(i % pieces) * VEC;
  float g[VEC], u[VEC], o[VEC];
  load_vec<VEC>(gate + row * gate_stride + c, g);
  load_vec<VEC>(up + row * up_stride + c, u);
#pragma unroll
  for (int e = 0; e < VEC; ++e) {
    if (UNIT != kClamped) {
      o[e] = (UNIT == kGelu ? gelu_tanh<T>(g[e]) : fmaxf(g[e], 0.f)) * u[e];
      continue;
    }
    const float gg = fminf(g[e], limit);
    const float uu = fminf(fmaxf(u[e], -limit), limit);
    o[e] = gg * sigmoid_for<T>(alpha * gg) * (uu + 1.0f);
  }
  store_vec<VEC>(out + row * out_stride + c, o);
}

template <GatedUnit UNIT>
static int launch_glu(const void* gate, int64_t gate_row_stride, const void* up, int64_t up_row_stride, void* out, int64_t out_row_stride, int dtype,
                      int64_t rows, int64_t n, float alpha, float limit, void* stream) {
  if (!known_dtype(dtype) || rows < 0 || n <= 0 || n > (1 << 24)) return MOPS_HIP_EINVAL;
  if (rows == 0) return MOPS_HIP_OK;
  if (!gate || !up || !out || gate_row_stride < n || up_row_stride < n || out_row_stride < n) return MOPS_HIP_EINVAL;
  const bool vec = n % 8 == 0 && gate_row_stride % 8 == 0 && up_row_stride % 8 == 0 && out_row_stride % 8 == 0 && aligned16(gate) && aligned16(up) && aligned16(out);
  const int64_t wgs = (rows * (n / (vec ? 8 : 1)) + 255) / 256;
  if (wgs > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  hipStream_t s = (hipStream_t)stream;
#define MOPS_GLU(T, V) hipLaunchKernelGGL((clamped_glu_kernel<T, V, UNIT>), dim3((unsigned)wgs), dim3(256), 0, s, (const T*)gate, gate_row_stride, \
                       (const T*)up, up_row_stride, (T*)out, out_row_stride, rows, (int)n, alpha, limit)
  if (dtype == MOPS_HIP_BF16) { if (vec) MOPS_GLU(bf16_t, 8); else MOPS_GLU(bf16_t, 1); }
  else { if (vec) MOPS_GLU(float, 8); else MOPS_GLU(float, 1); }
#undef MOPS_GLU
  return finish_launch();
}

}  // namespace mops

extern "C" int mops_hip_clamped_glu(const void* gate, int64_t gate_row_stride, const void* up, int64_t up_row_stride, void* out,
                                    int64_t out_row_stride, int dtype, int64_t rows, int64_t n, float alpha, float limit, void* stream) {
  return mops::launch_glu<mops::kClamped>(gate, gate_row_stride, up, up_row_stride, out, out_row_stride, dtype, rows, n, alpha, limit, stream);
}

extern "C" int mops_hip_gelu_glu(const void* gate, int64_t gate_row_stride, const void* up, int64_t up_row_stride, void* out,
                                 int64_t out_row_stride, int dtype, int64_t rows, int64_t n, void* stream) {
  return mops::launch_glu<mops::kGelu>(gate, gate_row_stride, up, up_row_stride, out, out_row_stride, dtype, rows, n, 0.f, 0.f, stream);
}

extern "C" int mops_hip_relu_glu(const void* gate, int64_t gate_row_stride, const void* up, int64_t up_row_stride, void* out,
                                 int64_t out_row_stride, int dtype, int64_t rows, int64_t n, void* stream) {
  return mops::launch_glu<mops::kRelu>(gate, gate_row_stride, up, up_row_stride, out, out_row_stride, dtype, rows, n, 0.f, 0.f, stream);
}
