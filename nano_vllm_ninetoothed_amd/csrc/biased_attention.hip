// Causal attention over paged keys and values with a linear distance bias per head:
//   score(i, j) = (q_i . k_j) * scale - slope_h (i - j),  j <= i,  softmax over j,  query head h reads key/value head h / (H / G).
// Instead of the bias a cap on the scores, or a bias rate_h ln(1 + step_h (i - j)), or no softmax at all: every key counts with
// sigmoid(score + bias_h).  Options: a window or chunks with kept first tokens (visible.h), a sink in the softmax's denominator, a gate
// per head or per element on the output, a constant factor.
// Key and value sizes are independent of each other; pages hold [block][offset][G][size rounded up to 8], zeros behind the size.
//
//   attention_prepare       from the packed projections [q | k | v] of every token: RMS norm with plain weights over the whole of
//                           q and over the whole of k, a factor per position on q, scatter of k and v into their pages
//   biased_attention_rows   one query row at a time, on vector units.  The plain form: any size, bf16 or float.
#include "visible.h"

namespace mops {

// One workgroup per token.  VEC = 8: the sizes are multiples of eight and nothing is padded.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void attention_prepare_kernel(const mops_hip_attention_prepare_args a) {
  __shared__ float scratch[4];
  const int64_t t = blockIdx.x;
  const int heads = (int)a.heads, groups = (int)a.kv_heads, dim = (int)a.dim, vdim = (int)a.vdim;
  const int dp = (dim + 7) / 8 * 8, vp = (vdim + 7) / 8 * 8, nq = heads * dim, nk = groups * dim;
  const T* row = (const T*)a.qkv + t * a.qkv_stride;
  auto square_sum = [&](const T* p, int n) {
    float ss = 0.f;
    for (int i = threadIdx.x * VEC; i < n; i += 256 * VEC) {
      float v[VEC];
      load_vec<VEC>(p + i, v);
#pragma unroll
      for (int e = 0; e < VEC; ++e) ss += v[e] * v[e];
    }
    return block_sum<256>(ss, scratch);
  };
  const float rq = 1.0f / sqrtf(square_sum(row, nq) / (float)nq + a.eps);
  const float rk = 1.0f / sqrtf(square_sum(row + nq, nk) / (float)nk + a.eps);
  auto write = [&](const T* src, const T* w, float factor, float factor2, T* dst, int n_heads, int size, int padded) {
    for (int i = threadIdx.x * VEC; i < n_heads * padded; i += 256 * VEC) {
      float v[VEC], wv[VEC];
      const int h = i / padded, d = i % padded;
      if (VEC > 1 || d < size) {
        load_vec<VEC>(src + h * size + d, v);
        if (w) {
          load_vec<VEC>(w + h * size + d, wv);
#pragma unroll
          for (int e = 0; e < VEC; ++e) v[e] = v[e] * factor * wv[e] * factor2;
        }
      } else {
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] = 0.f;
      }
      store_vec<VEC>(dst + i, v);
    }
  };
  int pos = a.positions[t];
  pos = pos < 0 ? 0 : (pos < a.max_positions ? pos : (int)a.max_positions - 1);
  write(row, (const T*)a.q_weight, rq, a.q_factor ? a.q_factor[pos] : 1.f, (T*)a.q + t * heads * dp, heads, dim, dp);
  const int64_t slot = a.slot_mapping[t];
  if (slot < 0 || slot >= a.num_slots) return;
  write(row + nq, (const T*)a.k_weight, rk, 1.f, (T*)a.k_pages + slot * groups * dp, groups, dim, dp);
  write(row + nq + nk, (const T*)nullptr, 1.f, 1.f, (T*)a.v_pages + slot * groups * vp, groups, vdim, vp);
}

constexpr int kRowKeys = 256;      // keys per pass
constexpr int kRowMaxDim = 2048, kRowMaxValue = 1024;

template <typename T>
__global__ __launch_bounds__(256) void biased_attention_rows_kernel(const mops_hip_biased_attention a) {
  __shared__ float sq[kRowMaxDim];
  __shared__ float sp[kRowKeys];
  __shared__ float red[4];
  const int h = blockIdx.x % (int)a.heads;
  const int64_t row = blockIdx.x / (int)a.heads;
  const int tid = threadIdx.x, ln = tid & 15, r16 = tid >> 4;
  const int dim = (int)a.dim, vdim = (int)a.vdim, groups = (int)a.kv_heads, g = h / (int)(a.heads / a.kv_heads);
  const int dp = (dim + 7) / 8 * 8, vp = (vdim + 7) / 8 * 8;
  T* out = (T*)a.out + row * a.out_stride + (int64_t)h * vdim;
  const int len = a.context_lens[row];
  if (len <= 0) {
    for (int i = tid; i < vdim; i += 256) out[i] = from_f32<T>(0.f);
    return;
  }
  const T* q = (const T*)a.q + (row * a.heads + h) * dp;
  for (int i = tid; i < dim; i += 256) sq[i] = to_f32(q[i]);
  const float slope = a.slopes ? a.slopes[h] : 0.f, rate = a.log_rate ? a.log_rate[h] : 0.f, step = a.log_rate ? a.log_step[h] : 0.f;
  const float bias = a.weight_bias ? a.weight_bias[h] : 0.f;
  const Visible see = visible_at(a, len);
  const int seq = a.row_seq ? a.row_seq[row] : (int)row;
  const int32_t* table = a.block_table + (int64_t)seq * a.block_table_stride;
  auto token_row = [&](int j) -> int64_t {      // the row of token j in the pages, -1 without one
    const int blk = j / (int)a.block_size;
    if (blk >= a.max_blocks) return -1;
    const int id = table[blk];
    return id < 0 || id >= a.num_blocks ? -1 : (int64_t)id * a.block_size + j % (int)a.block_size;
  };
  float m = a.sinks ? a.sinks[h] : -INFINITY, l = a.sinks ? 1.f : 0.f;      // a sink is a key with a value of zeros
  float acc[kRowMaxValue / 256];
#pragma unroll
  for (int i = 0; i < kRowMaxValue / 256; ++i) acc[i] = 0.f;
  for (int k0 = 0; k0 < len; k0 += kRowKeys) {
    if (k0 >= see.kept && k0 + kRowKeys <= see.lo) k0 = see.lo / kRowKeys * kRowKeys;      // nothing to see up to there
    __syncthreads();
    for (int kk = r16; kk < kRowKeys; kk += 16) {
      const int j = k0 + kk;
      const int64_t r = j < len && (j >= see.lo || j < see.kept) ? token_row(j) : -1;
      float dot = 0.f;
      if (r >= 0) {
        const T* kr = (const T*)a.k_pages + (r * groups + g) * dp;
        for (int i = ln; i < dim; i += 16) dot += sq[i] * to_f32(kr[i]);
      }
      dot = group_sum<16>(dot);
      if (ln == 0) {
        dot *= a.scale;
        if (a.softcap > 0.f) dot = a.softcap * tanhf(dot / a.softcap);
        if (a.log_rate) dot -= rate * log1pf(step * (float)(len - 1 - j));
        sp[kk] = r >= 0 ? dot - slope * (float)(len - 1 - j) + bias : -INFINITY;
      }
    }
    __syncthreads();
    float mx = group_max<kWave>(sp[tid]);
    if ((tid & 63) == 0) red[tid >> 6] = mx;
    __syncthreads();
    mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    const float m_new = fmaxf(m, mx);
    const float safe = m_new == -INFINITY ? 0.f : m_new;
    const float alpha = a.weight_bias ? 1.f : expf(m - safe);
    const float p = a.weight_bias ? 1.0f / (1.0f + expf(-sp[tid])) : expf(sp[tid] - safe);
    __syncthreads();
    sp[tid] = p;
    const float ps = group_sum<kWave>(p);
    if ((tid & 63) == 0) red[tid >> 6] = ps;
    __syncthreads();
    l = l * alpha + (red[0] + red[1]) + (red[2] + red[3]);
    m = m_new;
#pragma unroll
    for (int i = 0; i < kRowMaxValue / 256; ++i) acc[i] *= alpha;
    const int n = len - k0 < kRowKeys ? len - k0 : kRowKeys;
    for (int kk = 0; kk < n; ++kk) {
      const float w = sp[kk];
      const int64_t r = w != 0.f ? token_row(k0 + kk) : -1;
      if (r < 0) continue;
      const T* vr = (const T*)a.v_pages + (r * groups + g) * vp;
#pragma unroll
      for (int i = 0; i < kRowMaxValue / 256; ++i)
        if (tid + 256 * i < vdim) acc[i] += w * to_f32(vr[tid + 256 * i]);
    }
  }
  const float inv = a.weight_bias ? 1.0f : (l > 0.f ? 1.0f / l : 0.f);
  const OutputGate<T> gate(a, row, h);
#pragma unroll
  for (int i = 0; i < kRowMaxValue / 256; ++i)
    if (tid + 256 * i < vdim) out[tid + 256 * i] = from_f32<T>(acc[i] * inv * gate(tid + 256 * i));
}

// 1: go on; otherwise the status to return.
int check_biased_attention(const mops_hip_biased_attention* a) {
  if (!a || !known_dtype(a->dtype) || a->rows < 0) return MOPS_HIP_EINVAL;
  if (a->rows == 0) return MOPS_HIP_OK;
  if (!a->q || !a->k_pages || !a->v_pages || !a->context_lens || !a->block_table || !a->out) return MOPS_HIP_EINVAL;
  if (a->heads <= 0 || a->kv_heads <= 0 || a->heads % a->kv_heads || a->dim <= 0 || a->vdim <= 0) return MOPS_HIP_EINVAL;
  if (a->block_size <= 0 || a->num_blocks <= 0 || a->max_blocks <= 0 || a->block_table_stride < a->max_blocks) return MOPS_HIP_EINVAL;
  if (a->window < 0 || a->chunk < 0 || a->keep_first < 0 || (a->window && a->chunk)) return MOPS_HIP_EINVAL;
  if (!(a->softcap >= 0.f) || (a->gate && a->gate_stride < (a->gate_each ? a->heads * a->vdim : a->heads))) return MOPS_HIP_EINVAL;
  if ((a->softcap > 0.f) + (a->slopes != nullptr) + (a->log_rate != nullptr) + (a->weight_bias != nullptr) > 1) return MOPS_HIP_EINVAL;
  if ((a->log_rate == nullptr) != (a->log_step == nullptr) || (a->weight_bias && a->sinks) || (a->out_stride && a->out_stride < a->heads * a->vdim)) return MOPS_HIP_EINVAL;
  if (a->window > kMaxRange || a->chunk > kMaxRange || a->keep_first > kMaxRange) return MOPS_HIP_EUNSUPPORTED;
  if (a->rows * a->heads > 0x7fffffffLL || a->block_size > (1 << 20) || a->max_blocks * a->block_size > (1 << 28)) return MOPS_HIP_EUNSUPPORTED;
  return 1;
}

}  // namespace mops

extern "C" int mops_hip_attention_prepare(const mops_hip_attention_prepare_args* a, void* stream) {
  using namespace mops;
  if (!a || !known_dtype(a->dtype) || a->tokens < 0 || a->heads <= 0 || a->kv_heads <= 0 || a->dim <= 0 || a->vdim <= 0 || a->num_slots <= 0 ||
      a->max_positions <= 0)
    return MOPS_HIP_EINVAL;
  if (a->tokens == 0) return MOPS_HIP_OK;
  if (!a->qkv || !a->q_weight || !a->k_weight || !a->positions || !a->slot_mapping || !a->q || !a->k_pages || !a->v_pages) return MOPS_HIP_EINVAL;
  if (a->qkv_stride < (a->heads + a->kv_heads) * a->dim + a->kv_heads * a->vdim) return MOPS_HIP_EINVAL;
  if (a->tokens > 0x7fffffffLL || a->heads * a->dim > (1 << 20) || a->kv_heads * (a->dim + a->vdim) > (1 << 20)) return MOPS_HIP_EUNSUPPORTED;
  const bool vec = a->dim % 8 == 0 && a->vdim % 8 == 0 && a->qkv_stride % 8 == 0 && aligned16(a->qkv) && aligned16(a->q_weight) &&
                   aligned16(a->k_weight) && aligned16(a->q) && aligned16(a->k_pages) && aligned16(a->v_pages);
  const dim3 grid((unsigned)a->tokens);
  hipStream_t s = (hipStream_t)stream;
  if (a->dtype == MOPS_HIP_BF16) {
    if (vec) hipLaunchKernelGGL((attention_prepare_kernel<bf16_t, 8>), grid, dim3(256), 0, s, *a);
    else hipLaunchKernelGGL((attention_prepare_kernel<bf16_t, 1>), grid, dim3(256), 0, s, *a);
  } else {
    if (vec) hipLaunchKernelGGL((attention_prepare_kernel<float, 8>), grid, dim3(256), 0, s, *a);
    else hipLaunchKernelGGL((attention_prepare_kernel<float, 1>), grid, dim3(256), 0, s, *a);
  }
  return finish_launch();
}

extern "C" int mops_hip_biased_attention_rows(const mops_hip_biased_attention* a, void* stream) {
  using namespace mops;
  const int pre = check_biased_attention(a);
  if (pre != 1) return pre;
  if (a->dim > kRowMaxDim || a->vdim > kRowMaxValue) return MOPS_HIP_EUNSUPPORTED;
  const dim3 grid((unsigned)(a->rows * a->heads));
  if (a->dtype == MOPS_HIP_BF16) hipLaunchKernelGGL((biased_attention_rows_kernel<bf16_t>), grid, dim3(256), 0, (hipStream_t)stream, completed(*a));
  else hipLaunchKernelGGL((biased_attention_rows_kernel<float>), grid, dim3(256), 0, (hipStream_t)stream, completed(*a));
  return finish_launch();
}
