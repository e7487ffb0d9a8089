// A float32 residual stream and the norms around it, for models whose residual sum and norms are kept in 32 bits.
//
//   embed_residual     x = scale * table[id], as float32 (the residual) and in the activation type (the first projection's input)
//   norm_residual_add  x += rms(y) * (offset + w): the norm sits on the sublayer's output, the sum runs on in float32 and
//                      leaves a copy in the activation type for the next projection
//   rms_norm_f32       out = rms(x) * (offset + w) of the float32 stream
//   add_norm_norm      x += norm(y) * w_out, out = norm(x) * w_in: norms behind one sublayer and in front of the next, in one pass;
//                      RMS norms or layer norms
//   layer_norm_f32     out = (x - mean) / sqrt(variance + eps) * w of the float32 stream
//   add_norm           x += y + shift, or x = y + shift, then out = norm(x) * w + b (or x itself) in the activation type: a sublayer's
//                      output as it is, the norm in front of the next one
//   embed_pairs        embed_residual plus a row of a table of pairs of tokens
//   gated_group_norm   rms over equal parts of a row, with silu(gate) or sigmoid(gate) multiplied in before or after the division
//
// A row belongs to one workgroup of 64 or 256 threads; the elements a thread owns stay in its registers between the
// statistics and the scaling (up to kKeep pieces; longer rows read the rest again).
#include "mixed_types.h"

namespace mops {

constexpr int kKeep = 4;

template <typename T, int VEC>
__global__ __launch_bounds__(256) void embed_residual_kernel(const int64_t* __restrict__ ids, const T* __restrict__ table,
                                                             int64_t table_stride, float scale, float* __restrict__ x, T* __restrict__ act,
                                                             int64_t act_stride, int64_t vocab, int width) {
  const int64_t row = blockIdx.x;
  const int64_t id = ids[row];
  const bool ok = id >= 0 && id < vocab;
  for (int c = threadIdx.x * VEC; c < width; c += 256 * VEC) {
    float v[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = 0.f;
    if (ok) load_vec<VEC>(table + id * table_stride + c, v);
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] *= scale;
    store_vec<VEC>(x + row * width + c, v);
    if (act) store_vec<VEC>(act + row * act_stride + c, v);
  }
}

// The same plus a row of a table of pairs: (token in front * mul_prev + token * mul_cur) mod buckets, and row `buckets` for a
// sequence's first token.  The token in front of a portion is kept per state slot: the workgroup of the portion's first token is the
// only one that reads it, and it files the portion's last token behind its read.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void embed_pairs_kernel(const mops_hip_embed_pairs_args a) {
  const int64_t t = blockIdx.x;
  const int width = (int)a.width;
  const int64_t b = a.token_seq ? a.token_seq[t] : t;
  const int64_t first = a.cu_seqlens ? a.cu_seqlens[b] : t;
  const int64_t id = a.ids[t];
  int64_t pair = a.buckets, prev = -1;
  if (t > first) {
    prev = a.ids[t - 1];
  } else {
    const int slot = a.state_slots[b];
    const bool filed = slot >= 0 && slot < a.num_slots;
    if (filed && a.starts[b] > 0) prev = a.before[slot];
    __syncthreads();
    if (filed && threadIdx.x == 0) a.before[slot] = (int32_t)a.ids[a.cu_seqlens ? a.cu_seqlens[b + 1] - 1 : t];
  }
  if (prev >= 0) {
    pair = (prev * a.mul_prev + id * a.mul_cur) % a.buckets;
    if (pair < 0) pair += a.buckets;
  }
  const bool ok = id >= 0 && id < a.vocab;
  const T *row = (const T*)a.table + (ok ? id : 0) * a.table_stride, *row2 = (const T*)a.pairs + pair * a.pairs_stride;
  for (int c = threadIdx.x * VEC; c < width; c += 256 * VEC) {
    float v[VEC], u[VEC];
    load_vec<VEC>(row + c, v);
    load_vec<VEC>(row2 + c, u);
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = (ok ? a.scale * v[e] : 0.f) + u[e];
    store_vec<VEC>(a.residual + t * width + c, v);
  }
}

// MODE 0: out = norm(x) with x float32; MODE 1: residual += norm(y), out = the new residual in the activation type.
template <typename T, int VEC, int THREADS, int MODE>
__global__ __launch_bounds__(THREADS) void norm_kernel(float* __restrict__ residual, const T* __restrict__ y, int64_t y_stride,
                                                       const T* __restrict__ w, float offset, float eps, T* __restrict__ out,
                                                       int n) {
  __shared__ float scratch[THREADS / kWave];
  const int64_t row = blockIdx.x;
  float* xr = residual + row * n;
  const T* yr = y + row * y_stride;
  float keep[kKeep][VEC];
  float ss = 0.f;
#pragma unroll
  for (int it = 0; it < kKeep; ++it) {
    const int c = (it * THREADS + threadIdx.x) * VEC;
    if (c < n) {
      if (MODE == 0) load_vec<VEC>(xr + c, keep[it]);
      else load_vec<VEC>(yr + c, keep[it]);
#pragma unroll
      for (int e = 0; e < VEC; ++e) ss += keep[it][e] * keep[it][e];
    }
  }
  for (int c = (kKeep * THREADS + threadIdx.x) * VEC; c < n; c += THREADS * VEC) {
    float v[VEC];
    if (MODE == 0) load_vec<VEC>(xr + c, v);
    else load_vec<VEC>(yr + c, v);
#pragma unroll
    for (int e = 0; e < VEC; ++e) ss += v[e] * v[e];
  }
  const float rstd = 1.0f / sqrtf(block_sum<THREADS>(ss, scratch) / (float)n + eps);
  auto finish = [&](int c, const float (&v)[VEC]) {
    float wv[VEC], o[VEC];
    load_vec<VEC>(w + c, wv);
    if (MODE == 1) {
      load_vec<VEC>(xr + c, o);
#pragma unroll
      for (int e = 0; e < VEC; ++e) o[e] += v[e] * rstd * (offset + wv[e]);
      store_vec<VEC>(xr + c, o);
    } else {
#pragma unroll
      for (int e = 0; e < VEC; ++e) o[e] = v[e] * rstd * (offset + wv[e]);
    }
    store_vec<VEC>(out + row * n + c, o);
  };
#pragma unroll
  for (int it = 0; it < kKeep; ++it) {
    const int c = (it * THREADS + threadIdx.x) * VEC;
    if (c < n) finish(c, keep[it]);
  }
  for (int c = (kKeep * THREADS + threadIdx.x) * VEC; c < n; c += THREADS * VEC) {
    float v[VEC];
    if (MODE == 0) load_vec<VEC>(xr + c, v);
    else load_vec<VEC>(yr + c, v);
    finish(c, v);
  }
}

// residual += norm(sum of the row's `parts` rows of y, and of extra) * w_out; out = norm(residual) * w_in.  CENTER: the norms take
// the mean off first.
template <typename T, int VEC, int THREADS, bool CENTER>
__global__ __launch_bounds__(THREADS) void add_norm_norm_kernel(float* __restrict__ residual, const T* __restrict__ y, int64_t y_stride,
                                                                int parts, const T* __restrict__ extra, const T* __restrict__ w_out,
                                                                const T* __restrict__ w_in, float eps, T* __restrict__ out, int n) {
  __shared__ float scratch[THREADS / kWave];
  const int64_t row = blockIdx.x;
  float* xr = residual + row * n;
  const T* yr = y + row * parts * y_stride;
  auto read = [&](int c, float (&v)[VEC]) {
    load_vec<VEC>(yr + c, v);
    auto more = [&](const T* p) {
      float u[VEC];
      load_vec<VEC>(p + c, u);
#pragma unroll
      for (int e = 0; e < VEC; ++e) v[e] += u[e];
    };
    for (int p = 1; p < parts; ++p) more(yr + p * y_stride);
    if (extra) more(extra + row * n);
  };
  auto stream = [&](int c, float (&v)[VEC]) { load_vec<VEC>(xr + c, v); };      // this thread's own stores, once it has made them
  float keep[kKeep][VEC];
  // f(column, values) for all pieces of this thread; those behind the kept ones come from `again`
  auto each = [&](auto&& again, auto&& f) {
#pragma unroll
    for (int it = 0; it < kKeep; ++it) {
      const int c = (it * THREADS + threadIdx.x) * VEC;
      if (c < n) f(c, keep[it]);
    }
    for (int c = (kKeep * THREADS + threadIdx.x) * VEC; c < n; c += THREADS * VEC) {
      float v[VEC];
      again(c, v);
      f(c, v);
    }
  };
  // mean (0 without CENTER) and reciprocal root of the mean squared deviation from it
  auto statistics = [&](auto&& again, float sum, float squares, float& mean, float& rstd) {
    mean = 0.f;
    if (CENTER) {
      mean = block_sum<THREADS>(sum, scratch) / (float)n;
      squares = 0.f;
      each(again, [&](int, float (&v)[VEC]) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) squares += (v[e] - mean) * (v[e] - mean);
      });
    }
    rstd = 1.0f / sqrtf(block_sum<THREADS>(squares, scratch) / (float)n + eps);
  };
  float sum = 0.f, squares = 0.f, mean, rstd;
  auto count = [&](const float (&v)[VEC]) {
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      if (CENTER) sum += v[e];
      else squares += v[e] * v[e];
    }
  };
#pragma unroll
  for (int it = 0; it < kKeep; ++it) {
    const int c = (it * THREADS + threadIdx.x) * VEC;
    if (c < n) read(c, keep[it]);
  }
  each(read, [&](int, float (&v)[VEC]) { count(v); });
  statistics(read, sum, squares, mean, rstd);
  sum = squares = 0.f;
  each(read, [&](int c, float (&v)[VEC]) {      // v: the sublayer's output, then the new residual
    float wv[VEC], x[VEC];
    load_vec<VEC>(w_out + c, wv);
    load_vec<VEC>(xr + c, x);
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = x[e] + (v[e] - mean) * rstd * wv[e];
    store_vec<VEC>(xr + c, v);
    count(v);
  });
  statistics(stream, sum, squares, mean, rstd);
  each(stream, [&](int c, float (&v)[VEC]) {
    float wv[VEC], o[VEC];
    load_vec<VEC>(w_in + c, wv);
#pragma unroll
    for (int e = 0; e < VEC; ++e) o[e] = (v[e] - mean) * rstd * wv[e];
    store_vec<VEC>(out + row * n + c, o);
  });
}

// out = (x - mean) / sqrt(variance + eps) * w of the float32 stream.
template <typename T, int VEC, int THREADS>
__global__ __launch_bounds__(THREADS) void layer_norm_kernel(const float* __restrict__ x, const T* __restrict__ w, float eps, T* __restrict__ out, int n) {
  __shared__ float scratch[THREADS / kWave];
  const float* xr = x + (int64_t)blockIdx.x * n;
  float keep[kKeep][VEC];
  auto each = [&](auto&& f) {
#pragma unroll
    for (int it = 0; it < kKeep; ++it) {
      const int c = (it * THREADS + threadIdx.x) * VEC;
      if (c < n) f(c, keep[it]);
    }
    for (int c = (kKeep * THREADS + threadIdx.x) * VEC; c < n; c += THREADS * VEC) {
      float v[VEC];
      load_vec<VEC>(xr + c, v);
      f(c, v);
    }
  };
#pragma unroll
  for (int it = 0; it < kKeep; ++it) {
    const int c = (it * THREADS + threadIdx.x) * VEC;
    if (c < n) load_vec<VEC>(xr + c, keep[it]);
  }
  float sum = 0.f, squares = 0.f;
  each([&](int, float (&v)[VEC]) {
#pragma unroll
    for (int e = 0; e < VEC; ++e) sum += v[e];
  });
  const float mean = block_sum<THREADS>(sum, scratch) / (float)n;
  each([&](int, float (&v)[VEC]) {
#pragma unroll
    for (int e = 0; e < VEC; ++e) squares += (v[e] - mean) * (v[e] - mean);
  });
  const float rstd = 1.0f / sqrtf(block_sum<THREADS>(squares, scratch) / (float)n + eps);
  each([&](int c, float (&v)[VEC]) {
    float wv[VEC], o[VEC];
    load_vec<VEC>(w + c, wv);
#pragma unroll
    for (int e = 0; e < VEC; ++e) o[e] = (v[e] - mean) * rstd * wv[e];
    store_vec<VEC>(out + (int64_t)blockIdx.x * n + c, o);
  });
}

// residual += y + shift (or = y + shift; y and shift may be missing), out = norm(residual) * w + b, or the residual without w.
template <typename T, int VEC, int THREADS, bool CENTER>
__global__ __launch_bounds__(THREADS) void add_norm_kernel(const mops_hip_add_norm_args a) {
  __shared__ float scratch[THREADS / kWave];
  const int64_t row = blockIdx.x;
  const int n = (int)a.n;
  float* xr = a.residual + row * n;
  const T *yr = a.y ? (const T*)a.y + row * a.y_stride : nullptr, *w = (const T*)a.w, *b = (const T*)a.b;
  T* out = a.out ? (T*)a.out + row * a.out_stride : nullptr;
  float keep[kKeep][VEC];
  auto each = [&](auto&& f) {      // pieces behind the kept ones: this thread's own stores, once it has made them
#pragma unroll
    for (int it = 0; it < kKeep; ++it) {
      const int c = (it * THREADS + threadIdx.x) * VEC;
      if (c < n) f(c, keep[it]);
    }
    for (int c = (kKeep * THREADS + threadIdx.x) * VEC; c < n; c += THREADS * VEC) {
      float v[VEC];
      load_vec<VEC>(xr + c, v);
      f(c, v);
    }
  };
  auto read = [&](int c, float (&v)[VEC]) {
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = 0.f;
    if (!a.replace) load_vec<VEC>(xr + c, v);
    if (!yr && !a.shift) return;
    float u[VEC];
    if (yr) {
      load_vec<VEC>(yr + c, u);
#pragma unroll
      for (int e = 0; e < VEC; ++e) v[e] += u[e];
    }
    if (a.shift) {
      load_vec<VEC>(a.shift + c, u);
#pragma unroll
      for (int e = 0; e < VEC; ++e) v[e] += u[e];
    }
    store_vec<VEC>(xr + c, v);
  };
#pragma unroll
  for (int it = 0; it < kKeep; ++it) {
    const int c = (it * THREADS + threadIdx.x) * VEC;
    if (c < n) read(c, keep[it]);
  }
  for (int c = (kKeep * THREADS + threadIdx.x) * VEC; c < n; c += THREADS * VEC) {
    float v[VEC];
    read(c, v);
  }
  if (!out) return;
  float mean = 0.f, rstd = 1.f;
  if (w) {
    float sum = 0.f;
    if (CENTER) {
      each([&](int, float (&v)[VEC]) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) sum += v[e];
      });
      mean = block_sum<THREADS>(sum, scratch) / (float)n;
    }
    float squares = 0.f;
    each([&](int, float (&v)[VEC]) {
#pragma unroll
      for (int e = 0; e < VEC; ++e) squares += (v[e] - mean) * (v[e] - mean);
    });
    rstd = 1.0f / sqrtf(block_sum<THREADS>(squares, scratch) / (float)n + a.eps);
  }
  each([&](int c, float (&v)[VEC]) {
    float o[VEC], u[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) o[e] = (v[e] - mean) * rstd;
    if (w) {
      load_vec<VEC>(w + c, u);
#pragma unroll
      for (int e = 0; e < VEC; ++e) o[e] *= u[e];
    }
    if (b) {
      load_vec<VEC>(b + c, u);
#pragma unroll
      for (int e = 0; e < VEC; ++e) o[e] += u[e];
    }
    store_vec<VEC>(out + c, o);
  });
}

// LANES lanes per (row, part): parts of `size` consecutive elements.
template <typename T, int VEC, int LANES, bool GATE_FIRST>
__global__ __launch_bounds__(256) void gated_group_norm_kernel(const T* __restrict__ y, int64_t y_stride, const T* __restrict__ gate,
                                                               int64_t gate_stride, const T* __restrict__ w, bool shared_w, bool plain_sigmoid,
                                                               float eps, float scale, T* __restrict__ out, int64_t out_stride, int64_t rows,
                                                               int groups, int size) {
  const int64_t item = (int64_t)blockIdx.x * (256 / LANES) + threadIdx.x / LANES;
  if (item >= rows * groups) return;      // whole groups of lanes leave; the sums below stay inside a group
  const int lane = threadIdx.x & (LANES - 1);
  const int64_t row = item / groups;
  const int col0 = (int)(item % groups) * size;
  const T* yr = y + row * y_stride + col0;
  const T* gr = gate + row * gate_stride + col0;
  T* orow = out + row * out_stride + col0;
  if (w && !shared_w) w += col0;
  float keep[kKeep][VEC], gk[kKeep][VEC];
  float ss = 0.f;
  auto read = [&](int c, float (&v)[VEC], float (&g)[VEC]) {
    load_vec<VEC>(yr + c, v);
    load_vec<VEC>(gr + c, g);
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      g[e] = plain_sigmoid ? sigmoid_for<T>(g[e]) : silu_for<T>(g[e]);
      if (GATE_FIRST) v[e] *= g[e];
    }
  };
#pragma unroll
  for (int it = 0; it < kKeep; ++it) {
    const int c = (it * LANES + lane) * VEC;
    if (c < size) {
      read(c, keep[it], gk[it]);
#pragma unroll
      for (int e = 0; e < VEC; ++e) ss += keep[it][e] * keep[it][e];
    }
  }
  for (int c = (kKeep * LANES + lane) * VEC; c < size; c += LANES * VEC) {
    float v[VEC], g[VEC];
    read(c, v, g);
#pragma unroll
    for (int e = 0; e < VEC; ++e) ss += v[e] * v[e];
  }
  const float rstd = scale / sqrtf(group_sum<LANES>(ss) / (float)size + eps);
  auto finish = [&](int c, const float (&v)[VEC], const float (&g)[VEC]) {
    float o[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) o[e] = GATE_FIRST ? v[e] * rstd : v[e] * rstd * g[e];
    if (w) {
      float wv[VEC];
      load_vec<VEC>(w + c, wv);
#pragma unroll
      for (int e = 0; e < VEC; ++e) o[e] *= wv[e];
    }
    store_vec<VEC>(orow + c, o);
  };
#pragma unroll
  for (int it = 0; it < kKeep; ++it) {
    const int c = (it * LANES + lane) * VEC;
    if (c < size) finish(c, keep[it], gk[it]);
  }
  for (int c = (kKeep * LANES + lane) * VEC; c < size; c += LANES * VEC) {
    float v[VEC], g[VEC];
    read(c, v, g);
    finish(c, v, g);
  }
}

template <typename T, int MODE>
static void launch_norm(float* residual, const void* y, int64_t y_stride, const void* w, float offset, float eps, void* out,
                        int64_t rows, int64_t n, hipStream_t s) {
  const bool vec = n % 8 == 0 && y_stride % 8 == 0 && aligned16(residual) && (MODE == 0 || aligned16(y)) && aligned16(w) && aligned16(out);
  const dim3 grid((unsigned)rows);
#define MOPS_NORM(V, TH) hipLaunchKernelGGL((norm_kernel<T, V, TH, MODE>), grid, dim3(TH), 0, s, residual, (const T*)y, y_stride, \
                                            (const T*)w, offset, eps, (T*)out, (int)n)
  if (vec && n <= 1024) MOPS_NORM(8, 64);
  else if (vec) MOPS_NORM(8, 256);
  else if (n <= 512) MOPS_NORM(1, 64);
  else MOPS_NORM(1, 256);
#undef MOPS_NORM
}

}  // namespace mops

extern "C" int mops_hip_embed_residual(const int64_t* ids, const void* table, int64_t table_row_stride, int dtype, float scale,
                                       float* residual, void* act, int64_t act_stride, int64_t n_ids, int64_t vocab, int64_t width,
                                       void* stream) {
  using namespace mops;
  if (!known_dtype(dtype) || n_ids < 0 || vocab <= 0 || width <= 0 || width > (1 << 20) || n_ids > 0x7fffffffLL) return MOPS_HIP_EINVAL;
  if (n_ids == 0) return MOPS_HIP_OK;
  if (!ids || !table || !residual || table_row_stride < width || (act && act_stride < width)) return MOPS_HIP_EINVAL;
  const bool vec = width % 8 == 0 && table_row_stride % 8 == 0 && aligned16(table) && aligned16(residual) && (!act || (aligned16(act) && act_stride % 8 == 0));
  const dim3 grid((unsigned)n_ids), block(256);
  hipStream_t s = (hipStream_t)stream;
#define MOPS_EMBED(T, V) hipLaunchKernelGGL((embed_residual_kernel<T, V>), grid, block, 0, s, ids, (const T*)table, table_row_stride, \
                                            scale, residual, (T*)act, act_stride, vocab, (int)width)
  if (dtype == MOPS_HIP_BF16) { if (vec) MOPS_EMBED(bf16_t, 8); else MOPS_EMBED(bf16_t, 1); }
  else { if (vec) MOPS_EMBED(float, 8); else MOPS_EMBED(float, 1); }
#undef MOPS_EMBED
  return finish_launch();
}

extern "C" int mops_hip_norm_residual_add(float* residual, const void* y, int64_t y_row_stride, const void* weight, float weight_offset,
                                          float eps, void* act, int dtype, int64_t rows, int64_t n, void* stream) {
  using namespace mops;
  if (!known_dtype(dtype) || rows < 0 || n <= 0 || n > (1 << 20) || rows > 0x7fffffffLL) return MOPS_HIP_EINVAL;
  if (rows == 0) return MOPS_HIP_OK;
  if (!residual || !y || !weight || !act || y_row_stride < n || y == act) return MOPS_HIP_EINVAL;
  if (dtype == MOPS_HIP_BF16) launch_norm<bf16_t, 1>(residual, y, y_row_stride, weight, weight_offset, eps, act, rows, n, (hipStream_t)stream);
  else launch_norm<float, 1>(residual, y, y_row_stride, weight, weight_offset, eps, act, rows, n, (hipStream_t)stream);
  return finish_launch();
}

extern "C" int mops_hip_rms_norm_f32(const float* x, const void* weight, float weight_offset, float eps, void* out, int dtype,
                                     int64_t rows, int64_t n, void* stream) {
  using namespace mops;
  if (!known_dtype(dtype) || rows < 0 || n <= 0 || n > (1 << 20) || rows > 0x7fffffffLL) return MOPS_HIP_EINVAL;
  if (rows == 0) return MOPS_HIP_OK;
  if (!x || !weight || !out || (const void*)x == out) return MOPS_HIP_EINVAL;
  float* xr = const_cast<float*>(x);   // mode 0 only reads it
  if (dtype == MOPS_HIP_BF16) launch_norm<bf16_t, 0>(xr, nullptr, 0, weight, weight_offset, eps, out, rows, n, (hipStream_t)stream);
  else launch_norm<float, 0>(xr, nullptr, 0, weight, weight_offset, eps, out, rows, n, (hipStream_t)stream);
  return finish_launch();
}

extern "C" int mops_hip_add_norm_norm(float* residual, const void* y, int64_t y_row_stride, int64_t parts, const void* extra, const void* w_out,
                                      const void* w_in, float eps, int center, void* out, int dtype, int64_t rows, int64_t n, void* stream) {
  using namespace mops;
  if (!known_dtype(dtype) || rows < 0 || n <= 0 || n > (1 << 20) || rows > 0x7fffffffLL || parts <= 0 || parts > (1 << 20)) return MOPS_HIP_EINVAL;
  if (rows == 0) return MOPS_HIP_OK;
  if (!residual || !y || !w_out || !w_in || !out || y_row_stride < n || y == out || (extra && extra == out)) return MOPS_HIP_EINVAL;
  const bool vec = n % 8 == 0 && y_row_stride % 8 == 0 && aligned16(residual) && aligned16(y) && aligned16(w_out) && aligned16(w_in) && aligned16(out) &&
                   (!extra || aligned16(extra));
  const dim3 grid((unsigned)rows);
  hipStream_t s = (hipStream_t)stream;
#define MOPS_ANN(T, V, TH, C) hipLaunchKernelGGL((add_norm_norm_kernel<T, V, TH, C>), grid, dim3(TH), 0, s, residual, (const T*)y, y_row_stride, \
                                                 (int)parts, (const T*)extra, (const T*)w_out, (const T*)w_in, eps, (T*)out, (int)n)
#define MOPS_ANN_TYPE(T, C) do {                          \
    if (vec && n <= 1024) MOPS_ANN(T, 8, 64, C);          \
    else if (vec) MOPS_ANN(T, 8, 256, C);                 \
    else if (n <= 512) MOPS_ANN(T, 1, 64, C);             \
    else MOPS_ANN(T, 1, 256, C);                          \
  } while (0)
  if (dtype == MOPS_HIP_BF16) { if (center) MOPS_ANN_TYPE(bf16_t, true); else MOPS_ANN_TYPE(bf16_t, false); }
  else { if (center) MOPS_ANN_TYPE(float, true); else MOPS_ANN_TYPE(float, false); }
#undef MOPS_ANN_TYPE
#undef MOPS_ANN
  return finish_launch();
}

extern "C" int mops_hip_layer_norm_f32(const float* x, const void* weight, float eps, void* out, int dtype, int64_t rows, int64_t n, void* stream) {
  using namespace mops;
  if (!known_dtype(dtype) || rows < 0 || n <= 0 || n > (1 << 20) || rows > 0x7fffffffLL) return MOPS_HIP_EINVAL;
  if (rows == 0) return MOPS_HIP_OK;
  if (!x || !weight || !out || (const void*)x == out) return MOPS_HIP_EINVAL;
  const bool vec = n % 8 == 0 && aligned16(x) && aligned16(weight) && aligned16(out);
  const dim3 grid((unsigned)rows);
  hipStream_t s = (hipStream_t)stream;
#define MOPS_LN(T, V, TH) hipLaunchKernelGGL((layer_norm_kernel<T, V, TH>), grid, dim3(TH), 0, s, x, (const T*)weight, eps, (T*)out, (int)n)
#define MOPS_LN_TYPE(T) do {                          \
    if (vec && n <= 1024) MOPS_LN(T, 8, 64);          \
    else if (vec) MOPS_LN(T, 8, 256);                 \
    else if (n <= 512) MOPS_LN(T, 1, 64);             \
    else MOPS_LN(T, 1, 256);                          \
  } while (0)
  if (dtype == MOPS_HIP_BF16) MOPS_LN_TYPE(bf16_t);
  else MOPS_LN_TYPE(float);
#undef MOPS_LN_TYPE
#undef MOPS_LN
  return finish_launch();
}

extern "C" int mops_hip_add_norm(const mops_hip_add_norm_args* a, void* stream) {
  using namespace mops;
  if (!a || !known_dtype(a->dtype) || a->rows < 0 || a->n <= 0 || a->n > (1 << 20) || a->rows > 0x7fffffffLL) return MOPS_HIP_EINVAL;
  if (a->rows == 0) return MOPS_HIP_OK;
  if (!a->residual || (a->y && a->y_stride < a->n) || (a->out && a->out_stride < a->n) || (a->y && a->y == a->out) || (a->b && !a->w) ||
      (a->replace && !a->y && !a->shift))
    return MOPS_HIP_EINVAL;
  auto good = [](const void* p) { return !p || aligned16(p); };
  const bool vec = a->n % 8 == 0 && (!a->y || a->y_stride % 8 == 0) && (!a->out || a->out_stride % 8 == 0) && good(a->residual) && good(a->y) &&
                   good(a->shift) && good(a->w) && good(a->b) && good(a->out);
  const dim3 grid((unsigned)a->rows);
  hipStream_t s = (hipStream_t)stream;
#define MOPS_AN(T, V, TH, C) hipLaunchKernelGGL((add_norm_kernel<T, V, TH, C>), grid, dim3(TH), 0, s, *a)
#define MOPS_AN_TYPE(T, C) do {                          \
    if (vec && a->n <= 1024) MOPS_AN(T, 8, 64, C);       \
    else if (vec) MOPS_AN(T, 8, 256, C);                 \
    else if (a->n <= 512) MOPS_AN(T, 1, 64, C);          \
    else MOPS_AN(T, 1, 256, C);                          \
  } while (0)
  if (a->dtype == MOPS_HIP_BF16) { if (a->center) MOPS_AN_TYPE(bf16_t, true); else MOPS_AN_TYPE(bf16_t, false); }
  else { if (a->center) MOPS_AN_TYPE(float, true); else MOPS_AN_TYPE(float, false); }
#undef MOPS_AN_TYPE
#undef MOPS_AN
  return finish_launch();
}

extern "C" int mops_hip_embed_pairs(const mops_hip_embed_pairs_args* a, void* stream) {
  using namespace mops;
  if (!a || !known_dtype(a->dtype) || a->tokens < 0 || a->vocab <= 0 || a->width <= 0 || a->width > (1 << 20) || a->buckets <= 0 || a->num_slots <= 0)
    return MOPS_HIP_EINVAL;
  if (a->tokens == 0) return MOPS_HIP_OK;
  if (!a->ids || !a->table || !a->pairs || !a->residual || !a->before || !a->starts || !a->state_slots) return MOPS_HIP_EINVAL;
  if (a->table_stride < a->width || a->pairs_stride < a->width || (a->token_seq == nullptr) != (a->cu_seqlens == nullptr)) return MOPS_HIP_EINVAL;
  const int64_t most = 0x7fffffffLL;      // products of token ids and factors stay inside 64 bits
  if (a->tokens > most || a->vocab > most || a->mul_prev > most || a->mul_cur > most || a->mul_prev < -most || a->mul_cur < -most) return MOPS_HIP_EUNSUPPORTED;
  const bool vec = a->width % 8 == 0 && a->table_stride % 8 == 0 && a->pairs_stride % 8 == 0 && aligned16(a->table) && aligned16(a->pairs) && aligned16(a->residual);
  const dim3 grid((unsigned)a->tokens), block(256);
  hipStream_t s = (hipStream_t)stream;
#define MOPS_PAIRS(T, V) hipLaunchKernelGGL((embed_pairs_kernel<T, V>), grid, block, 0, s, *a)
  if (a->dtype == MOPS_HIP_BF16) { if (vec) MOPS_PAIRS(bf16_t, 8); else MOPS_PAIRS(bf16_t, 1); }
  else { if (vec) MOPS_PAIRS(float, 8); else MOPS_PAIRS(float, 1); }
#undef MOPS_PAIRS
  return finish_launch();
}

extern "C" int mops_hip_gated_group_norm(const void* y, int64_t y_row_stride, const void* gate, int64_t gate_row_stride,
                                         const void* weight, int shared_weight, float eps, int gate_first, int plain_sigmoid, float scale,
                                         void* out, int64_t out_row_stride, int dtype, int64_t rows, int64_t groups, int64_t group_size,
                                         void* stream) {
  using namespace mops;
  if (!known_dtype(dtype) || rows < 0 || groups <= 0 || group_size <= 0 || groups * group_size > (1 << 24)) return MOPS_HIP_EINVAL;
  if (rows == 0) return MOPS_HIP_OK;
  const int64_t n = groups * group_size;
  if (!y || !gate || !out || y_row_stride < n || gate_row_stride < n || out_row_stride < n || out == gate) return MOPS_HIP_EINVAL;
  const bool vec = group_size % 8 == 0 && out_row_stride % 8 == 0 && y_row_stride % 8 == 0 && gate_row_stride % 8 == 0 && aligned16(y) && aligned16(gate) &&
                   aligned16(out) && (!weight || aligned16(weight));
  const bool small = vec && group_size <= 64, narrow = group_size <= 512;      // eight lanes, a row of lanes, a wave per group
  const int64_t per_wg = small ? 32 : (narrow ? 16 : 4), wgs = (rows * groups + per_wg - 1) / per_wg;
  if (wgs > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  hipStream_t s = (hipStream_t)stream;
#define MOPS_GGN(T, V, L, F) hipLaunchKernelGGL((gated_group_norm_kernel<T, V, L, F>), dim3((unsigned)wgs), dim3(256), 0, s, (const T*)y, \
                          y_row_stride, (const T*)gate, gate_row_stride, (const T*)weight, shared_weight != 0, plain_sigmoid != 0, eps, scale, \
                          (T*)out, out_row_stride, rows, (int)groups, (int)group_size)
#define MOPS_GGN2(T, V) do {                                    \
    if (V == 8 && small) { if (gate_first) MOPS_GGN(T, V, 8, true); else MOPS_GGN(T, V, 8, false); }  \
    else if (narrow) { if (gate_first) MOPS_GGN(T, V, 16, true); else MOPS_GGN(T, V, 16, false); }  \
    else { if (gate_first) MOPS_GGN(T, V, 64, true); else MOPS_GGN(T, V, 64, false); }         \
  } while (0)
  if (dtype == MOPS_HIP_BF16) { if (vec) MOPS_GGN2(bf16_t, 8); else MOPS_GGN2(bf16_t, 1); }
  else { if (vec) MOPS_GGN2(float, 8); else MOPS_GGN2(float, 1); }
#undef MOPS_GGN2
#undef MOPS_GGN
  return finish_launch();
}
