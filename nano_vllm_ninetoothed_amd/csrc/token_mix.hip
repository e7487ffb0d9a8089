// What a time-mixing layer does in front of its projections and its recurrence.
//
//   token_mix        out[p][t] = x[t] + (x[t-1] - x[t]) * mu[p] for several vectors mu at once: every token is moved some way
//                    towards the token in front of it.  The row in front of a portion comes from one row per state slot (zeros
//                    at the start of a sequence), which receives the last row of the portion.
//   low_rank_decay   out[t, c] = -exp(sum_r w2[c, r] tanh(z[t, r]) + w0[c]): the natural logarithm of a decay per channel, float32; or
//                    with a rate per head out[t, c] = rate[head of c] softplus(sum_r w2[c, r] z[t, r] + w0[c])
#include "mfma_tiles.h"

namespace mops {

// A thread owns VEC channels of a token.  The thread of a portion's first token is the only one that reads the slot's row, and
// it also writes it, behind its read.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void token_mix_kernel(const T* __restrict__ x, int64_t x_stride, const float* __restrict__ mu, int parts,
                                                        T* __restrict__ before, int64_t num_slots, const int32_t* __restrict__ token_seq,
                                                        const int32_t* __restrict__ cu_seqlens, const int32_t* __restrict__ starts,
                                                        const int32_t* __restrict__ state_slots, T* __restrict__ out, int64_t tokens,
                                                        int width) {
  const int pieces = width / VEC;
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= tokens * pieces) return;
  const int64_t t = i / pieces;
  const int c = (int)(i % pieces) * VEC;
  const int64_t b = token_seq ? token_seq[t] : t;
  const int64_t first = cu_seqlens ? cu_seqlens[b] : t;
  float v[VEC], prev[VEC];
  load_vec<VEC>(x + t * x_stride + c, v);
  if (t > first) {
    load_vec<VEC>(x + (t - 1) * x_stride + c, prev);
  } else {
#pragma unroll
    for (int e = 0; e < VEC; ++e) prev[e] = 0.f;
    const int slot = state_slots[b];
    if (slot >= 0 && slot < num_slots) {
      T* row = before + (int64_t)slot * width + c;
      if (starts[b] > 0) load_vec<VEC>(row, prev);
      const int64_t last = cu_seqlens ? cu_seqlens[b + 1] - 1 : t;
      float u[VEC];
      load_vec<VEC>(x + last * x_stride + c, u);
      store_vec<VEC>(row, u);
    }
  }
#pragma unroll
  for (int e = 0; e < VEC; ++e) prev[e] -= v[e];
  for (int p = 0; p < parts; ++p) {
    float m[VEC];
    load_vec<VEC>(mu + (int64_t)p * width + c, m);
#pragma unroll
    for (int e = 0; e < VEC; ++e) m[e] = v[e] + prev[e] * m[e];
    store_vec<VEC>(out + ((int64_t)p * tokens + t) * width + c, m);
  }
}

constexpr int kDecayChannels = 256, kDecayMaxRank = 256;

// tanh with an absolute error of about 1e-7, far below what its rounding to bf16 costs any but the smallest values
__device__ __forceinline__ float tanh_fast(float v) {
  return 1.0f - 2.0f * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(2.8853900817779268f * v));
}

// Workgroup = 16 TT tokens x 256 channels, a wave takes 64 of the channels; tanh(z) (with RATED z) in LDS, the rows of w2 straight from
// memory.
template <int TT, bool RATED>
__global__ __launch_bounds__(256) void low_rank_decay_mfma_kernel(const uint16_t* __restrict__ z, int64_t z_stride, const uint16_t* __restrict__ w2,
                                                                  const float* __restrict__ w0, const float* __restrict__ rate, int head_size,
                                                                  float* __restrict__ out, int64_t tokens, int channels, int rank, bool aligned, bool z_aligned, bool wide) {
  constexpr int kDecayTokens = 16 * TT;
  extern __shared__ __align__(16) unsigned char smem[];
  uint16_t* const tile = reinterpret_cast<uint16_t*>(smem);
  const int ksteps = (rank + 31) / 32, pitch = ksteps * 32 + 8;
  const int64_t t0 = (int64_t)blockIdx.x * kDecayTokens;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, n = lane & 15, jj = lane >> 4;
  const int c0 = blockIdx.y * kDecayChannels + wave * 64;
  auto weights = [&](int i, int ks) {
    const int c = c0 + 16 * i + n;
    return c < channels ? load8_guarded(w2 + (int64_t)c * rank, 32 * ks + 8 * jj, rank, aligned) : u32x4{0u, 0u, 0u, 0u};
  };
  u32x4 first[4];      // on their way while the tile is filled
#pragma unroll
  for (int i = 0; i < 4; ++i) first[i] = weights(i, 0);
  for (int i = threadIdx.x; i < kDecayTokens * ksteps * 4; i += 256) {
    const int r = i / (ksteps * 4), k = i % (ksteps * 4) * 8;
    u32x4 w = {0u, 0u, 0u, 0u};
    if (t0 + r < tokens) w = load8_guarded(z + (t0 + r) * z_stride, k, rank, z_aligned);
    if (!RATED) {
#pragma unroll
      for (int e = 0; e < 4; ++e) w[e] = pack_bf16x2(tanh_fast(bf16lo_to_f32(w[e])), tanh_fast(bf16hi_to_f32(w[e])));
    }
    store16(tile + r * pitch + k, w);
  }
  __syncthreads();
  f32x4 acc[4][TT];      // [channels][tokens]
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < TT; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int ks = 0; ks < ksteps; ++ks) {
    bf16x8 b[TT];
#pragma unroll
    for (int j = 0; j < TT; ++j) b[j] = tile_row(tile, pitch, 16 * j + n, 32 * ks + 8 * jj);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const u32x4 a = ks == 0 ? first[i] : weights(i, ks);
#pragma unroll
      for (int j = 0; j < TT; ++j) acc[i][j] = mfma16(__builtin_bit_cast(bf16x8, a), b[j], acc[i][j]);
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int c = c0 + 16 * i + 4 * jj;
    float bias[4], per[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      bias[e] = c + e < channels ? w0[c + e] : 0.f;
      per[e] = RATED && c + e < channels ? rate[(c + e) / head_size] : 0.f;
    }
#pragma unroll
    for (int j = 0; j < TT; ++j) {
      const int64_t t = t0 + 16 * j + n;
      if (t >= tokens) continue;
      f32x4 o;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float x = acc[i][j][e] + bias[e];
        o[e] = RATED ? per[e] * softplus_fast(x) : -__builtin_amdgcn_exp2f(1.4426950408889634f * x);
      }
      float* dst = out + t * channels + c;
      if (wide && c + 4 <= channels) {
        *reinterpret_cast<f32x4*>(dst) = o;
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (c + e < channels) dst[e] = o[e];
      }
    }
  }
}

constexpr int kDecayPlainRank = 4096;

template <typename T>
__global__ __launch_bounds__(256) void low_rank_decay_kernel(const T* __restrict__ z, int64_t z_stride, const T* __restrict__ w2,
                                                             const float* __restrict__ w0, const float* __restrict__ rate, int head_size,
                                                             float* __restrict__ out, int64_t tokens, int channels, int rank) {
  __shared__ float th[kDecayPlainRank];
  const int64_t t = blockIdx.x;
  for (int r = threadIdx.x; r < rank; r += 256) {
    const float x = to_f32(z[t * z_stride + r]);
    th[r] = rate ? x : tanhf(x);
  }
  __syncthreads();
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= channels) return;
  float acc = w0[c];
  for (int r = 0; r < rank; ++r) acc += to_f32(w2[(int64_t)c * rank + r]) * th[r];
  out[t * channels + c] = rate ? rate[c / head_size] * softplus_f32(acc) : -expf(acc);
}

}  // namespace mops

extern "C" int mops_hip_token_mix(const void* x, int64_t x_row_stride, const float* mu, int64_t parts, void* before, int64_t num_slots,
                                  const int32_t* token_seq, const int32_t* cu_seqlens, const int32_t* starts, const int32_t* state_slots,
                                  void* out, int dtype, int64_t tokens, int64_t width, void* stream) {
  using namespace mops;
  if (!known_dtype(dtype) || tokens < 0 || width <= 0 || width > (1 << 20) || parts <= 0 || parts > 64 || num_slots <= 0) return MOPS_HIP_EINVAL;
  if (tokens == 0) return MOPS_HIP_OK;
  if (!x || !mu || !before || !starts || !state_slots || !out || x_row_stride < width || !token_seq != !cu_seqlens) return MOPS_HIP_EINVAL;
  const bool vec = width % 8 == 0 && x_row_stride % 8 == 0 && aligned16(x) && aligned16(mu) && aligned16(before) && aligned16(out);
  const int64_t wgs = (tokens * (width / (vec ? 8 : 1)) + 255) / 256;
  if (wgs > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
#define MOPS_MIX(T, V) hipLaunchKernelGGL((token_mix_kernel<T, V>), dim3((unsigned)wgs), dim3(256), 0, (hipStream_t)stream, (const T*)x, x_row_stride, mu, \
                       (int)parts, (T*)before, num_slots, token_seq, cu_seqlens, starts, state_slots, (T*)out, tokens, (int)width)
  if (dtype == MOPS_HIP_BF16) { if (vec) MOPS_MIX(bf16_t, 8); else MOPS_MIX(bf16_t, 1); }
  else { if (vec) MOPS_MIX(float, 8); else MOPS_MIX(float, 1); }
#undef MOPS_MIX
  return finish_launch();
}

extern "C" int mops_hip_low_rank_decay(const void* z, int64_t z_row_stride, const void* w2, const float* w0, const float* rate, int64_t head_size,
                                       float* out, int dtype, int64_t tokens, int64_t channels, int64_t rank, void* stream) {
  using namespace mops;
  if (!known_dtype(dtype) || tokens < 0 || channels <= 0 || channels > (1 << 22) || rank <= 0) return MOPS_HIP_EINVAL;
  if (tokens == 0) return MOPS_HIP_OK;
  if (!z || !w2 || !w0 || !out || z_row_stride < rank || (rate && head_size <= 0)) return MOPS_HIP_EINVAL;
  if (rank > kDecayPlainRank || tokens > 0x7fffffffLL || (channels + 255) / 256 > 65535) return MOPS_HIP_EUNSUPPORTED;
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MOPS_HIP_BF16 && rank <= kDecayMaxRank) {
    const int per = tokens <= 2048 ? 16 : 64;
    const dim3 grid((unsigned)((tokens + per - 1) / per), (unsigned)((channels + kDecayChannels - 1) / kDecayChannels));
    const size_t lds = per * ((rank + 31) / 32 * 32 + 8) * 2;
    const bool w_aligned = rank % 8 == 0 && aligned16(w2), z_aligned = z_row_stride % 8 == 0 && aligned16(z), wide = channels % 4 == 0 && aligned16(out);
#define MOPS_LRM2(TT, R) hipLaunchKernelGGL((low_rank_decay_mfma_kernel<TT, R>), grid, dim3(256), lds, s, (const uint16_t*)z, z_row_stride, \
                                        (const uint16_t*)w2, w0, rate, (int)head_size, out, tokens, (int)channels, (int)rank, w_aligned, z_aligned, wide)
#define MOPS_LRM(TT) do { if (rate) MOPS_LRM2(TT, true); else MOPS_LRM2(TT, false); } while (0)
    if (per == 16) MOPS_LRM(1);
    else MOPS_LRM(4);
#undef MOPS_LRM
#undef MOPS_LRM2
    return finish_launch();
  }
  const dim3 grid((unsigned)tokens, (unsigned)((channels + 255) / 256));
#define MOPS_LRD(T) hipLaunchKernelGGL((low_rank_decay_kernel<T>), grid, dim3(256), 0, s, (const T*)z, z_row_stride, (const T*)w2, w0, rate, (int)head_size, out, \
                                       tokens, (int)channels, (int)rank)
  if (dtype == MOPS_HIP_BF16) MOPS_LRD(bf16_t);
  else MOPS_LRD(float);
#undef MOPS_LRD
  return finish_launch();
}
