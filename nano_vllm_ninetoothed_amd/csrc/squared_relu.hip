// squared_relu: out = max(x, 0)^2 over [rows, n].
#include "mixed_types.h"

namespace mops {

template <typename T, int VEC>
__global__ __launch_bounds__(256) void squared_relu_kernel(const T* __restrict__ x, int64_t x_stride, T* __restrict__ out, int64_t rows, int n) {
  const int pieces = n / VEC;
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= rows * pieces) return;
  const int64_t row = i / pieces;
  const int c = (int)(i % pieces) * VEC;
  float v[VEC];
  load_vec<VEC>(x + row * x_stride + c, v);
#pragma unroll
  for (int e = 0; e < VEC; ++e) {
    const float p = fmaxf(v[e], 0.f);
    v[e] = p * p;
  }
  store_vec<VEC>(out + row * n + c, v);
}

}  // namespace mops

extern "C" int mops_hip_squared_relu(const void* x, int64_t x_row_stride, void* out, int dtype, int64_t rows, int64_t n, void* stream) {
  using namespace mops;
  if (!known_dtype(dtype) || rows < 0 || n <= 0 || n > (1 << 24)) return MOPS_HIP_EINVAL;
  if (rows == 0) return MOPS_HIP_OK;
  if (!x || !out || x_row_stride < n) return MOPS_HIP_EINVAL;
  const bool vec = n % 8 == 0 && x_row_stride % 8 == 0 && aligned16(x) && aligned16(out);
  const int64_t wgs = (rows * (n / (vec ? 8 : 1)) + 255) / 256;
  if (wgs > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
#define MOPS_SR(T, V) hipLaunchKernelGGL((squared_relu_kernel<T, V>), dim3((unsigned)wgs), dim3(256), 0, (hipStream_t)stream, (const T*)x, x_row_stride, \
                                         (T*)out, rows, (int)n)
  if (dtype == MOPS_HIP_BF16) { if (vec) MOPS_SR(bf16_t, 8); else MOPS_SR(bf16_t, 1); }
  else { if (vec) MOPS_SR(float, 8); else MOPS_SR(float, 1); }
#undef MOPS_SR
  return finish_launch();
}
