// The gated delta rule, carried from token to token in float32:
//
//   S <- diag(e^g) S,  u = sigmoid(b) (v - S^T k),  S <- S + k u^T,  o = S^T q
//
// S is [d x vd] per head, kept transposed in memory as in decayed_recurrence.hip: state[slot][head][vd][pitch].  g is a logarithm per
// token, head and key channel.  q and k become unit vectors per head, q is multiplied by q_scale behind that; query/key heads may be
// shared by heads / groups consecutive value heads.
//
// delta_rule_kernel runs the tokens of a sequence one after the other with the state in registers: the decode step (with the short
// convolutions in front of q, k and v fused in), the float32 path, and the path of head sizes that delta_chunks.hip does not cover.
// Workgroup = (sequence, head, 16 RPT value rows); sixteen lanes share a row of the state, so that both products with it are sums
// over sixteen lanes.
#include "mixed_types.h"

namespace mops {

template <typename T, int DPT, int RPT, bool CONV>
__global__ __launch_bounds__(256) void delta_rule_kernel(const mops_hip_delta a, const int pitch) {
  constexpr int kRows = 16 * RPT, kDim = 16 * DPT, kPiece = DPT >= 4 ? 4 : DPT;
  __shared__ __align__(16) float sq[kDim], sk[kDim], sa[kDim], sv[kRows];
  __shared__ float scratch[4];
  const int heads = (int)a.heads, d = (int)a.d, vd = (int)a.vd, taps = (int)a.taps;
  const int tiles = (vd + kRows - 1) / kRows;
  const int tile = blockIdx.x % tiles, h = (blockIdx.x / tiles) % heads, b = blockIdx.x / (tiles * heads);
  const int t_begin = a.cu_seqlens ? a.cu_seqlens[b] : b, t_end = a.cu_seqlens ? a.cu_seqlens[b + 1] : b + 1;
  if (t_end <= t_begin) return;
  const int slot = a.state_slots[b], start = a.starts[b];
  const int row0 = tile * kRows, tid = threadIdx.x, ln = tid & 15, r16 = tid >> 4;
  T* out = (T*)a.out + (int64_t)h * vd + row0;
  if (slot < 0 || slot >= a.num_slots) {      // a padding row of a captured batch
    for (int t = t_begin; t < t_end; ++t)
      if (tid < kRows && row0 + tid < vd) out[t * a.out_stride + tid] = from_f32<T>(0.f);
    return;
  }
  float* state = a.state + (((int64_t)slot * heads + h) * vd + row0) * pitch;
  auto piece_at = [&](int p) { return p * 16 * kPiece + ln * kPiece; };
  float s[RPT][DPT];
#pragma unroll
  for (int r = 0; r < RPT; ++r)
#pragma unroll
    for (int p = 0; p < DPT / kPiece; ++p) {
      const int row = r16 + 16 * r, i = piece_at(p);
      float v[kPiece];
#pragma unroll
      for (int e = 0; e < kPiece; ++e) v[e] = 0.f;
      if (start > 0 && row0 + row < vd && i < pitch) load_vec<kPiece>(state + (int64_t)row * pitch + i, v);
#pragma unroll
      for (int e = 0; e < kPiece; ++e) s[r][p * kPiece + e] = v[e];
    }
  const int per_group = heads / (int)a.groups, g = h / per_group;
  const T *q = (const T*)a.q + (int64_t)g * d, *k = (const T*)a.k + (int64_t)g * d, *v = (const T*)a.v + (int64_t)h * vd + row0;
  T* ring = CONV ? (T*)a.conv_ring + (int64_t)slot * taps * a.channels : nullptr;
  // channel c of the convolution, current input x: the output for position start; `keep` also files x in the ring
  const int ring_row = CONV ? start % taps : 0, lags = start < taps - 1 ? start : taps - 1;
  auto conv = [&](float x, int64_t c, bool keep) {
    float acc = a.conv_weight[(int64_t)(taps - 1) * a.channels + c] * x;
#pragma unroll 4
    for (int lag = 1; lag <= lags; ++lag) {
      const int row = ring_row - lag < 0 ? ring_row - lag + taps : ring_row - lag;
      acc += a.conv_weight[(int64_t)(taps - 1 - lag) * a.channels + c] * to_f32(ring[(int64_t)row * a.channels + c]);
    }
    if (keep) ring[(int64_t)ring_row * a.channels + c] = from_f32<T>(x);
    return silu_for<T>(acc);
  };
  for (int t = t_begin; t < t_end; ++t) {
    float q_squares = 0.f, k_squares = 0.f;
    for (int j = tid; j < 2 * kDim; j += 256) {      // q, then k
      const bool is_k = j >= kDim;
      const int i = is_k ? j - kDim : j;
      float x = 0.f;
      if (i < d) {
        x = to_f32((is_k ? k + t * a.k_stride : q + t * a.q_stride)[i]);
        if (CONV) x = conv(x, (is_k ? a.k_channel : a.q_channel) + (int64_t)g * d + i, tile == 0 && h % per_group == 0);
      }
      (is_k ? sk : sq)[i] = x;
      (is_k ? k_squares : q_squares) += x * x;
    }
    for (int i = tid; i < kDim; i += 256) sa[i] = i < d ? expf(a.log_decay[t * a.log_decay_stride + (int64_t)h * d + i]) : 1.f;
    for (int i = tid; i < kRows; i += 256) {
      float x = 0.f;
      if (row0 + i < vd) {
        x = to_f32(v[t * a.v_stride + i]);
        if (CONV) x = conv(x, a.v_channel + (int64_t)h * vd + row0 + i, true);
      }
      sv[i] = x;
    }
    const float beta = sigmoid_for<float>(to_f32(((const T*)a.beta)[t * a.beta_stride + h]));
    const float rq = a.q_scale / sqrtf(block_sum<256>(q_squares, scratch) + a.unit_eps);
    const float rk = 1.0f / sqrtf(block_sum<256>(k_squares, scratch) + a.unit_eps);      // two barriers each: the tables are written
    float qq[DPT], kk[DPT], aa[DPT];
#pragma unroll
    for (int p = 0; p < DPT / kPiece; ++p)
#pragma unroll
      for (int e = 0; e < kPiece; ++e) {
        qq[p * kPiece + e] = sq[piece_at(p) + e] * rq;
        kk[p * kPiece + e] = sk[piece_at(p) + e] * rk;
        aa[p * kPiece + e] = sa[piece_at(p) + e];
      }
#pragma unroll
    for (int r = 0; r < RPT; ++r) {
      const int row = r16 + 16 * r;
      float seen = 0.f;
#pragma unroll
      for (int e = 0; e < DPT; ++e) {
        s[r][e] *= aa[e];
        seen += s[r][e] * kk[e];
      }
      const float u = beta * (sv[row] - group_sum<16>(seen));
      float dot = 0.f;
#pragma unroll
      for (int e = 0; e < DPT; ++e) {
        s[r][e] += kk[e] * u;
        dot += s[r][e] * qq[e];
      }
      dot = group_sum<16>(dot);
      if (ln == 0 && row0 + row < vd) out[t * a.out_stride + row] = from_f32<T>(dot);
    }
    __syncthreads();
  }
#pragma unroll
  for (int r = 0; r < RPT; ++r)
#pragma unroll
    for (int p = 0; p < DPT / kPiece; ++p) {
      const int row = r16 + 16 * r, i = piece_at(p);
      if (row0 + row >= vd || i >= pitch) continue;
      float v[kPiece];
#pragma unroll
      for (int e = 0; e < kPiece; ++e) v[e] = s[r][p * kPiece + e];
      store_vec<kPiece>(state + (int64_t)row * pitch + i, v);
    }
}

template <typename T, int DPT, bool CONV>
static void launch_delta_rows(const mops_hip_delta& a, hipStream_t s) {
  const int pitch = (int)mops_hip_recurrence_state_pitch(a.d);
#define MOPS_DELTA(R)                                                                                                    \
  hipLaunchKernelGGL((delta_rule_kernel<T, DPT, R, CONV>), dim3((unsigned)(a.batch * a.heads * ((a.vd + 16 * (R) - 1) / (16 * (R))))), dim3(256), 0, \
                     s, a, pitch)
  if (a.vd <= 16) MOPS_DELTA(1);
  else if (a.vd <= 32) MOPS_DELTA(2);
  else MOPS_DELTA(4);
#undef MOPS_DELTA
}

template <typename T, int DPT>
static void launch_delta_conv(const mops_hip_delta& a, hipStream_t s) {
  if (a.conv_weight) launch_delta_rows<T, DPT, true>(a, s);
  else launch_delta_rows<T, DPT, false>(a, s);
}

template <typename T>
static int launch_delta(const mops_hip_delta& a, hipStream_t s) {
  if (a.d <= 32) launch_delta_conv<T, 2>(a, s);
  else if (a.d <= 64) launch_delta_conv<T, 4>(a, s);
  else if (a.d <= 128) launch_delta_conv<T, 8>(a, s);
  else if (a.d <= 256) launch_delta_conv<T, 16>(a, s);
  else launch_delta_conv<T, 32>(a, s);
  return finish_launch();
}

// 1: go on; otherwise the status to return.
int check_delta(const mops_hip_delta* a) {
  if (!a || !known_dtype(a->dtype) || a->batch < 0) return MOPS_HIP_EINVAL;
  if (a->batch == 0) return MOPS_HIP_OK;
  if (!a->q || !a->k || !a->v || !a->out || !a->state || !a->state_slots || !a->starts || !a->log_decay || !a->beta) return MOPS_HIP_EINVAL;
  if (a->heads <= 0 || a->groups <= 0 || a->heads % a->groups || a->d <= 0 || a->vd <= 0 || a->num_slots <= 0) return MOPS_HIP_EINVAL;
  if (a->q_stride < a->groups * a->d || a->k_stride < a->groups * a->d || a->v_stride < a->heads * a->vd || a->out_stride < a->heads * a->vd ||
      a->log_decay_stride < a->heads * a->d || a->beta_stride < a->heads)
    return MOPS_HIP_EINVAL;
  if (a->d > 512 || a->heads > 65535 || a->vd > 65536 || a->batch > 65535) return MOPS_HIP_EUNSUPPORTED;
  if (!aligned16(a->state)) return MOPS_HIP_EALIGN;
  return 1;
}

}  // namespace mops

extern "C" int mops_hip_delta_rule(const mops_hip_delta* a, void* stream) {
  using namespace mops;
  const int pre = check_delta(a);
  if (pre != 1) return pre;
  if (a->conv_weight && (a->cu_seqlens || !a->conv_ring || a->taps <= 0 || a->channels <= 0 || a->q_channel < 0 || a->k_channel < 0 || a->v_channel < 0 ||
                         a->q_channel + a->groups * a->d > a->channels || a->k_channel + a->groups * a->d > a->channels ||
                         a->v_channel + a->heads * a->vd > a->channels))
    return MOPS_HIP_EINVAL;
  if (a->batch * a->heads * ((a->vd + 15) / 16) > 0x7fffffffLL || a->taps > 1024) return MOPS_HIP_EUNSUPPORTED;
  return a->dtype == MOPS_HIP_BF16 ? launch_delta<bf16_t>(*a, (hipStream_t)stream) : launch_delta<float>(*a, (hipStream_t)stream);
}
