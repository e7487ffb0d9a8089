// Latent attention over a paged cache that holds, per token, one latent row c (kv_rank values) and one rotated key part
// shared by all heads (rot_dim values): cache[block][offset][pitch] = [c | key part | zeros].
//
//   latent_prepare         from the down projections [query latent | kv latent | key part] of every token: RMS norm with plain
//                          weights of both latents, rotation of the key part (pairs (2i, 2i+1)), scatter of the cache row
//   head_linear            y[t, h, :] = W[h] x[t, h, :]: the per-head products that move a query into the latent space and a
//                          latent result out of it
//   latent_attention_rows  one query row at a time against the cache, in the latent space: the key of a head is
//                          [W_uk[h]^T q | q_rot] . [c | key part], the value is c.  Plain form: any size, bf16 or float.
#include "mfma_tiles.h"

namespace mops {

// One wave per (token, part): part 0 the query latent, part 1 the cache row.
template <typename T>
__global__ __launch_bounds__(128) void latent_prepare_kernel(const T* __restrict__ down, int64_t down_stride, const T* __restrict__ q_weight,
                                                             const T* __restrict__ kv_weight, float eps, const float* __restrict__ cos_sin,
                                                             int64_t max_positions, const int32_t* __restrict__ positions,
                                                             const int32_t* __restrict__ slot_mapping, T* __restrict__ cq,
                                                             T* __restrict__ cache, int64_t num_slots, int q_rank, int kv_rank, int rot,
                                                             int pitch) {
  const int64_t t = blockIdx.x;
  const int lane = threadIdx.x & (kWave - 1);
  const T* row = down + t * down_stride;
  if (threadIdx.x < kWave) {
    float ss = 0.f;
    for (int i = lane; i < q_rank; i += kWave) {
      const float v = to_f32(row[i]);
      ss += v * v;
    }
    const float rstd = 1.0f / sqrtf(group_sum<kWave>(ss) / (float)q_rank + eps);
    for (int i = lane; i < q_rank; i += kWave) cq[t * q_rank + i] = from_f32<T>(to_f32(row[i]) * rstd * to_f32(q_weight[i]));
    return;
  }
  const int64_t slot = slot_mapping[t];
  if (slot < 0 || slot >= num_slots) return;
  row += q_rank;
  T* dst = cache + slot * pitch;
  float ss = 0.f;
  for (int i = lane; i < kv_rank; i += kWave) {
    const float v = to_f32(row[i]);
    ss += v * v;
  }
  const float rstd = 1.0f / sqrtf(group_sum<kWave>(ss) / (float)kv_rank + eps);
  for (int i = lane; i < kv_rank; i += kWave) dst[i] = from_f32<T>(to_f32(row[i]) * rstd * to_f32(kv_weight[i]));
  int pos = positions[t];
  if (pos >= max_positions) pos = (int)max_positions - 1;
  const float* trig = cos_sin + (int64_t)pos * rot;
  for (int i = lane; i < rot / 2; i += kWave) {
    const float u = to_f32(row[kv_rank + 2 * i]), v = to_f32(row[kv_rank + 2 * i + 1]);
    const float c = trig[i], s = trig[rot / 2 + i];
    dst[kv_rank + 2 * i] = from_f32<T>(u * c - v * s);
    dst[kv_rank + 2 * i + 1] = from_f32<T>(v * c + u * s);
  }
  for (int i = kv_rank + rot + lane; i < pitch; i += kWave) dst[i] = from_f32<T>(0.f);
}

// Wave = 16 tokens x 64 outputs; the four waves of a workgroup take four token tiles against the same weights.
__global__ __launch_bounds__(256) void head_linear_bf16_kernel(const uint16_t* __restrict__ x, int64_t x_token_stride, int64_t x_head_stride,
                                                               const uint16_t* __restrict__ w, uint16_t* __restrict__ y,
                                                               int64_t y_token_stride, int64_t y_head_stride, int tokens, int k_size,
                                                               int n_size, bool aligned, bool wide_store) {
  const int lane = threadIdx.x & (kWave - 1);
  const int col = lane & 15, quad = lane >> 4;
  const int t = (blockIdx.x * 4 + threadIdx.x / kWave) * 16 + col;
  const int n0 = blockIdx.y * 64;
  const int h = blockIdx.z;
  const uint16_t* xr = x + (int64_t)(t < tokens ? t : 0) * x_token_stride + h * x_head_stride;
  const uint16_t* wh = w + (int64_t)h * n_size * k_size;
  f32x4 acc[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < k_size; k0 += 32) {
    const int kk = k0 + 8 * quad;
    const u32x4 b = load8_guarded(xr, kk, k_size, aligned);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int n = n0 + 16 * i + col;
      const u32x4 a = n < n_size ? load8_guarded(wh + (int64_t)n * k_size, kk, k_size, aligned) : u32x4{0u, 0u, 0u, 0u};
      acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), acc[i], 0, 0, 0);
    }
  }
  if (t >= tokens) return;
  uint16_t* yr = y + (int64_t)t * y_token_stride + h * y_head_stride;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int n = n0 + 16 * i + 4 * quad;
    if (wide_store && n + 4 <= n_size) {
      *reinterpret_cast<u32x2*>(yr + n) = u32x2{pack_bf16x2(acc[i][0], acc[i][1]), pack_bf16x2(acc[i][2], acc[i][3])};
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (n + e < n_size) yr[n + e] = (uint16_t)f32_to_bf16_bits(acc[i][e]);
    }
  }
}

__global__ __launch_bounds__(64) void head_linear_f32_kernel(const float* __restrict__ x, int64_t x_token_stride, int64_t x_head_stride,
                                                             const float* __restrict__ w, float* __restrict__ y, int64_t y_token_stride,
                                                             int64_t y_head_stride, int tokens, int k_size, int n_size) {
  const int n = blockIdx.y * 64 + threadIdx.x;
  const int t0 = blockIdx.x * 4;
  const int h = blockIdx.z;
  if (n >= n_size) return;
  const float* wr = w + ((int64_t)h * n_size + n) * k_size;
  float acc[4] = {0.f, 0.f, 0.f, 0.f};
  for (int k = 0; k < k_size; ++k) {
    const float wv = wr[k];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = t0 + i < tokens ? t0 + i : tokens - 1;
      acc[i] += wv * x[(int64_t)t * x_token_stride + h * x_head_stride + k];
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
    if (t0 + i < tokens) y[(int64_t)(t0 + i) * y_token_stride + h * y_head_stride + n] = acc[i];
}

constexpr int kRowKeys = 256;      // keys per pass of the plain form
constexpr int kRowMaxWidth = 2048; // kv_rank + rot_dim
constexpr int kRowMaxRank = 1024;

template <typename T>
__global__ __launch_bounds__(256) void latent_attention_rows_kernel(const mops_hip_latent_rows a) {
  __shared__ float sq[kRowMaxWidth];
  __shared__ float sp[kRowKeys];
  __shared__ float red[4];
  const int h = blockIdx.x % (int)a.heads;
  const int64_t row = blockIdx.x / (int)a.heads;
  const int tid = threadIdx.x, ln = tid & 15, r16 = tid >> 4;
  const int kv_rank = (int)a.kv_rank, rot = (int)a.rot_dim, width = kv_rank + rot;
  T* out = (T*)a.out + (row * a.heads + h) * kv_rank;
  const int len = a.context_lens[row];
  if (len <= 0) {
    for (int i = tid; i < kv_rank; i += 256) out[i] = from_f32<T>(0.f);
    return;
  }
  const T* ql = (const T*)a.q_latent + (row * a.heads + h) * kv_rank;
  const T* qr = (const T*)a.q_rot + row * a.q_rot_token_stride + h * a.q_rot_head_stride;
  int pos = len - 1;
  const float* trig = a.cos_sin + (int64_t)(pos < a.max_positions ? pos : a.max_positions - 1) * rot;
  for (int i = tid; i < kv_rank; i += 256) sq[i] = to_f32(ql[i]);
  for (int i = tid; i < rot / 2; i += 256) {
    const float u = to_f32(qr[2 * i]), v = to_f32(qr[2 * i + 1]);
    const float c = trig[i], s = trig[rot / 2 + i];
    sq[kv_rank + 2 * i] = u * c - v * s;
    sq[kv_rank + 2 * i + 1] = v * c + u * s;
  }
  const int seq = a.row_seq ? a.row_seq[row] : (int)row;
  const int32_t* table = a.block_table + (int64_t)seq * a.block_table_stride;
  auto key_row = [&](int j) -> const T* {
    const int blk = j / (int)a.block_size;
    if (blk >= a.max_blocks) return nullptr;
    const int id = table[blk];
    if (id < 0 || id >= a.num_blocks) return nullptr;
    return (const T*)a.cache + ((int64_t)id * a.block_size + j % (int)a.block_size) * a.pitch;
  };
  float m = -INFINITY, l = 0.f;
  float acc[kRowMaxRank / 256];
#pragma unroll
  for (int i = 0; i < kRowMaxRank / 256; ++i) acc[i] = 0.f;
  for (int k0 = 0; k0 < len; k0 += kRowKeys) {
    __syncthreads();
    for (int kk = r16; kk < kRowKeys; kk += 16) {
      const int j = k0 + kk;
      const T* kr = j < len ? key_row(j) : nullptr;
      float dot = 0.f;
      if (kr)
        for (int i = ln; i < width; i += 16) dot += sq[i] * to_f32(kr[i]);
      dot = group_sum<16>(dot);
      if (ln == 0) sp[kk] = kr ? dot * a.scale : -INFINITY;
    }
    __syncthreads();
    float mx = group_max<kWave>(sp[tid]);
    if ((tid & 63) == 0) red[tid >> 6] = mx;
    __syncthreads();
    mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    const float m_new = fmaxf(m, mx);
    const float safe = m_new == -INFINITY ? 0.f : m_new;
    const float alpha = expf(m - safe);
    const float p = expf(sp[tid] - safe);
    __syncthreads();
    sp[tid] = p;
    const float ps = group_sum<kWave>(p);
    if ((tid & 63) == 0) red[tid >> 6] = ps;
    __syncthreads();
    l = l * alpha + (red[0] + red[1]) + (red[2] + red[3]);
    m = m_new;
#pragma unroll
    for (int i = 0; i < kRowMaxRank / 256; ++i) acc[i] *= alpha;
    const int n = len - k0 < kRowKeys ? len - k0 : kRowKeys;
    for (int kk = 0; kk < n; ++kk) {
      const T* kr = key_row(k0 + kk);
      if (!kr) continue;
      const float w = sp[kk];
#pragma unroll
      for (int i = 0; i < kRowMaxRank / 256; ++i)
        if (tid + 256 * i < kv_rank) acc[i] += w * to_f32(kr[tid + 256 * i]);
    }
  }
  const float inv = l > 0.f ? 1.0f / l : 0.f;
#pragma unroll
  for (int i = 0; i < kRowMaxRank / 256; ++i)
    if (tid + 256 * i < kv_rank) out[tid + 256 * i] = from_f32<T>(acc[i] * inv);
}

int check_latent_rows(const mops_hip_latent_rows* a) {
  if (!a || !known_dtype(a->dtype) || a->rows < 0) return MOPS_HIP_EINVAL;
  if (a->rows == 0) return MOPS_HIP_OK;
  if (!a->q_latent || !a->q_rot || !a->cache || !a->cos_sin || !a->context_lens || !a->block_table || !a->out) return MOPS_HIP_EINVAL;
  if (a->heads <= 0 || a->kv_rank <= 0 || a->rot_dim < 0 || (a->rot_dim & 1) || a->pitch < a->kv_rank + a->rot_dim) return MOPS_HIP_EINVAL;
  if (a->block_size <= 0 || a->num_blocks <= 0 || a->max_blocks <= 0 || a->block_table_stride < a->max_blocks || a->max_positions <= 0)
    return MOPS_HIP_EINVAL;
  if (a->rows * a->heads > 0x7fffffffLL || a->block_size > (1 << 20)) return MOPS_HIP_EUNSUPPORTED;
  return 1;
}

}  // namespace mops

extern "C" int mops_hip_latent_prepare(const void* down, int64_t down_stride, const void* q_weight, const void* kv_weight, float eps,
                                       const float* cos_sin, int64_t max_positions, const int32_t* positions, const int32_t* slot_mapping,
                                       void* q_latent, void* cache, int64_t num_slots, int64_t pitch, int dtype, int64_t tokens,
                                       int64_t q_rank, int64_t kv_rank, int64_t rot_dim, void* stream) {
  using namespace mops;
  if (!known_dtype(dtype) || tokens < 0 || q_rank <= 0 || kv_rank <= 0 || rot_dim < 0 || (rot_dim & 1) || pitch < kv_rank + rot_dim ||
      num_slots <= 0 || max_positions <= 0)
    return MOPS_HIP_EINVAL;
  if (tokens == 0) return MOPS_HIP_OK;
  if (!down || !q_weight || !kv_weight || !cos_sin || !positions || !slot_mapping || !q_latent || !cache ||
      down_stride < q_rank + kv_rank + rot_dim)
    return MOPS_HIP_EINVAL;
  if (tokens > 0x7fffffffLL || pitch > (1 << 20) || q_rank > (1 << 20)) return MOPS_HIP_EUNSUPPORTED;
  const dim3 grid((unsigned)tokens), block(128);
  hipStream_t s = (hipStream_t)stream;
#define MOPS_PREP(T) hipLaunchKernelGGL((latent_prepare_kernel<T>), grid, block, 0, s, (const T*)down, down_stride, (const T*)q_weight,        \
                        (const T*)kv_weight, eps, cos_sin, max_positions, positions, slot_mapping, (T*)q_latent, (T*)cache, num_slots, (int)q_rank, \
                        (int)kv_rank, (int)rot_dim, (int)pitch)
  if (dtype == MOPS_HIP_BF16) MOPS_PREP(bf16_t);
  else MOPS_PREP(float);
#undef MOPS_PREP
  return finish_launch();
}

extern "C" int mops_hip_head_linear(const void* x, int64_t x_token_stride, int64_t x_head_stride, const void* w, void* y,
                                    int64_t y_token_stride, int64_t y_head_stride, int dtype, int64_t tokens, int64_t heads, int64_t n,
                                    int64_t k, void* stream) {
  using namespace mops;
  if (!known_dtype(dtype) || tokens < 0 || heads <= 0 || n <= 0 || k <= 0) return MOPS_HIP_EINVAL;
  if (tokens == 0) return MOPS_HIP_OK;
  if (!x || !w || !y || x_head_stride < 0 || y_head_stride < 0 || x_token_stride < 0 || y_token_stride < 0) return MOPS_HIP_EINVAL;
  if (tokens > (1 << 24) || heads > 65535 || n > (1 << 20) || k > (1 << 20)) return MOPS_HIP_EUNSUPPORTED;
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MOPS_HIP_BF16) {
    const bool aligned = k % 8 == 0 && x_token_stride % 8 == 0 && x_head_stride % 8 == 0 && aligned16(x) && aligned16(w);
    const bool wide = y_token_stride % 4 == 0 && y_head_stride % 4 == 0 && aligned16(y);
    const dim3 grid((unsigned)((tokens + 63) / 64), (unsigned)((n + 63) / 64), (unsigned)heads);
    hipLaunchKernelGGL(head_linear_bf16_kernel, grid, dim3(256), 0, s, (const uint16_t*)x, x_token_stride, x_head_stride, (const uint16_t*)w,
                       (uint16_t*)y, y_token_stride, y_head_stride, (int)tokens, (int)k, (int)n, aligned, wide);
  } else {
    const dim3 grid((unsigned)((tokens + 3) / 4), (unsigned)((n + 63) / 64), (unsigned)heads);
    hipLaunchKernelGGL(head_linear_f32_kernel, grid, dim3(64), 0, s, (const float*)x, x_token_stride, x_head_stride, (const float*)w, (float*)y,
                       y_token_stride, y_head_stride, (int)tokens, (int)k, (int)n);
  }
  return finish_launch();
}

extern "C" int mops_hip_latent_attention_rows(const mops_hip_latent_rows* a, void* stream) {
  using namespace mops;
  const int pre = check_latent_rows(a);
  if (pre != 1) return pre;
  if (a->kv_rank > kRowMaxRank || a->kv_rank + a->rot_dim > kRowMaxWidth) return MOPS_HIP_EUNSUPPORTED;
  const dim3 grid((unsigned)(a->rows * a->heads));
  if (a->dtype == MOPS_HIP_BF16) hipLaunchKernelGGL((latent_attention_rows_kernel<bf16_t>), grid, dim3(256), 0, (hipStream_t)stream, *a);
  else hipLaunchKernelGGL((latent_attention_rows_kernel<float>), grid, dim3(256), 0, (hipStream_t)stream, *a);
  return finish_launch();
}
