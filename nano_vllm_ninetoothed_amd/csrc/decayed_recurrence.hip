// Linear recurrences with one decay per head (or key channel) and token, carried from token to token in float32:
//
//   S_t = a_t S_(t-1) + k_t (s_t v_t)^T        S is [d x vd] per head, kept transposed in memory: state[slot][head][vd][pitch]
//   o_t = S_t^T q_t + skip v_t
//
// Ways to the decay a and the input scale s:
//   constant      a = decay[head], s = 1                                     (linear attention with a fixed decay)
//   time steps    s = softplus(dt + dt_bias[head]), a = exp(neg_a[head] s)   (state-space layers; skip = D[head])
//   per channel   S_t = diag(exp(channel_decay_t)) S_(t-1) + k_t v_t^T, channel_decay a float logarithm per token, head and key
//                 channel; the output looks at the state in front of the token and weighs the token itself by a bonus u per
//                 channel: o_t = (S_(t-1) + diag(u) k_t v_t^T)^T q_t
//   matrix memory a = exp(f + m_(t-1) - m_t), s = exp(i - m_t) with gates i = cap tanh((x + bias) / cap) and f = log sigmoid(cap tanh((y +
//                 bias) / cap)) per token and head, relative to a running maximum m_t = max(f + m_(t-1), i) that starts at 0; the same
//                 recurrence with values of one gives n, and o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6).  k_scale multiplies q instead.  n follows the value
//                 rows of a head's state, once per 64 of them, and so does m in `top`: every workgroup has a copy of its own.
// q and k may be rotated on their first rot dimensions (dimension i with i + rot/2) by the row of a cos/sin table, and k is
// multiplied by k_scale after that.  Query/key heads may be shared by heads / groups consecutive value heads.
//
// decayed_recurrence_kernel runs the tokens of a sequence one after the other with the state in registers.  It is the
// decode step (one token per sequence, optionally with the short convolution in front of q, k and v fused in), the
// float32 path, and the path of head sizes the chunked kernels do not cover.
//   workgroup = (sequence, head, tile of 16*RPT value rows): sixteen lanes share a row of the state, each lane holds
//   4-element pieces of it, so a row is read and written as 256-byte runs and the dot product with q is a sum over
//   sixteen lanes.
//
// short_conv: causal convolution per channel over the last `taps` tokens, bias and silu, for packed portions of sequences.
// The inputs before a portion come from a ring of `taps` rows per state slot, indexed by position modulo taps: a decode step
// reads the taps-1 rows before its own position and writes its own row, which is none of those, so the step needs no
// second buffer and no shifting.  Positions before the start of the sequence count as zeros whatever the ring holds.
// short_conv_update writes the last taps-1 inputs of each portion into the ring, in a launch of its own behind the readers.
#include "matrix_memory.h"

namespace mops {

struct RecurrenceArgs {
  const void *q, *k, *v;
  int64_t q_stride, k_stride, v_stride;
  void* out;
  int64_t out_stride;
  float* state;
  int64_t num_slots;
  const int32_t *state_slots, *cu_seqlens, *starts;
  int heads, groups, d, vd, pitch;
  const float* decay;
  const void* dt;
  int64_t dt_stride;
  const float *dt_bias, *neg_a, *skip;
  const float *channel_decay, *bonus;
  int64_t channel_decay_stride;
  const void *input_gate, *forget_gate;
  int64_t gate_stride;
  const float *input_bias, *forget_bias;
  float gate_cap;
  float* top;
  int copies;                   // of n and m: 0 without a matrix memory
  const float* cos_sin;
  int rot;
  int64_t max_positions;
  float k_scale;
  const float *conv_w, *conv_b;
  void* ring;
  int taps;
  int64_t channels;
  int q_channel, k_channel, v_channel;
};

enum RecurrenceKind { kPlain, kConvolved, kPerChannel, kMemory };

// cu_seqlens == nullptr: sequence b is the single token b.
template <typename T, int DPT, int RPT, RecurrenceKind KIND>
__global__ __launch_bounds__(256) void decayed_recurrence_kernel(const RecurrenceArgs a) {
  constexpr bool CONV = KIND == kConvolved, CHANNEL = KIND == kPerChannel, MEMORY = KIND == kMemory;
  constexpr int kRows = 16 * RPT;
  constexpr int kDim = 16 * DPT;
  __shared__ __align__(16) float sq[kDim], sk[kDim], sv[kRows], sa[CHANNEL ? kDim : 1], su[CHANNEL ? kDim : 1];
  const int tiles = (a.vd + kRows - 1) / kRows;
  const int tile = blockIdx.x % tiles;
  const int h = (blockIdx.x / tiles) % a.heads;
  const int b = blockIdx.x / (tiles * a.heads);
  const int t_begin = a.cu_seqlens ? a.cu_seqlens[b] : b;
  const int t_end = a.cu_seqlens ? a.cu_seqlens[b + 1] : b + 1;
  if (t_end <= t_begin) return;
  const int slot = a.state_slots[b];
  const int start = a.starts[b];
  const int row0 = tile * kRows;
  const int tid = threadIdx.x, ln = tid & 15, r16 = tid >> 4;
  T* out = (T*)a.out + (int64_t)h * a.vd + row0;
  if (slot < 0 || slot >= a.num_slots) {   // a padding row of a captured batch
    for (int t = t_begin; t < t_end; ++t)
      if (tid < kRows && row0 + tid < a.vd) out[t * a.out_stride + tid] = from_f32<T>(0.f);
    return;
  }
  float* const head_state = a.state + ((int64_t)slot * a.heads + h) * (a.vd + (MEMORY ? a.copies : 0)) * a.pitch;
  float* const state = head_state + (int64_t)row0 * a.pitch;
  float* const n_row = head_state + (int64_t)(a.vd + tile) * a.pitch;            // MEMORY
  float* const top = MEMORY ? a.top + ((int64_t)slot * a.heads + h) * a.copies + tile : nullptr;
  float s[RPT][DPT];
  constexpr int kPiece = DPT >= 4 ? 4 : DPT;
  auto piece_at = [&](int p) { return p * 64 + ln * kPiece; };
#pragma unroll
  for (int r = 0; r < RPT; ++r) {
    const int row = r16 + 16 * r;
#pragma unroll
    for (int p = 0; p < DPT / kPiece; ++p) {
      const int i = piece_at(p);
#pragma unroll
      for (int e = 0; e < kPiece; ++e) s[r][p * kPiece + e] = 0.f;
      if (start > 0 && row0 + row < a.vd && i < a.pitch) {
        float v[kPiece];
        if (kPiece == 4) load_vec<kPiece>(state + (int64_t)row * a.pitch + i, v);
        else {
#pragma unroll
          for (int e = 0; e < kPiece; ++e) v[e] = state[(int64_t)row * a.pitch + i + e];
        }
#pragma unroll
        for (int e = 0; e < kPiece; ++e) s[r][p * kPiece + e] = v[e];
      }
    }
  }
  float nn[MEMORY ? DPT : 1], m = 0.f;
  if (MEMORY) {
    if (start > 0) m = *top;
#pragma unroll
    for (int p = 0; p < DPT / kPiece; ++p)
#pragma unroll
      for (int e = 0; e < kPiece; ++e) {
        const int i = piece_at(p) + e;
        nn[MEMORY ? p * kPiece + e : 0] = start > 0 && i < a.pitch ? n_row[i] : 0.f;
      }
  }
  const int per_group = a.heads / a.groups;
  const int g = h / per_group;
  const T *q = (const T*)a.q + (int64_t)g * a.d, *k = (const T*)a.k + (int64_t)g * a.d, *v = (const T*)a.v + (int64_t)h * a.vd + row0;
  const float const_decay = a.decay ? a.decay[h] : 0.f;
  const float bias = a.dt ? a.dt_bias[h] : 0.f, neg_a = a.dt ? a.neg_a[h] : 0.f, skip = a.skip ? a.skip[h] : 0.f;
  // channel c of the convolution, current input x: the output for position pos; `keep` also files x in the ring
  T* ring = CONV ? (T*)a.ring + (int64_t)slot * a.taps * a.channels : nullptr;
  auto conv = [&](float x, int64_t c, int pos, bool keep) {
    float acc = a.conv_b[c] + a.conv_w[(int64_t)(a.taps - 1) * a.channels + c] * x;
    for (int lag = 1; lag < a.taps; ++lag)
      if (pos - lag >= 0)
        acc += a.conv_w[(int64_t)(a.taps - 1 - lag) * a.channels + c] * to_f32(ring[(int64_t)((pos - lag) % a.taps) * a.channels + c]);
    if (keep) ring[(int64_t)(pos % a.taps) * a.channels + c] = from_f32<T>(x);
    return silu_for<T>(acc);
  };
  for (int t = t_begin; t < t_end; ++t) {
    const int pos = start + (t - t_begin);
    const float* trig = a.rot ? a.cos_sin + (int64_t)(pos < a.max_positions ? pos : a.max_positions - 1) * a.rot : nullptr;
    const int half = a.rot >> 1;
    for (int i = tid; i < kDim; i += 256) {
      float qv = 0.f, kv = 0.f;
      if (i < a.d) {
        qv = to_f32(q[t * a.q_stride + i]);
        kv = to_f32(k[t * a.k_stride + i]);
        if (CONV) {
          const bool keep = tile == 0 && h % per_group == 0;
          qv = conv(qv, (int64_t)a.q_channel + g * a.d + i, pos, keep);
          kv = conv(kv, (int64_t)a.k_channel + g * a.d + i, pos, keep);
        }
        if (i < a.rot) {
          const bool lower = i < half;
          const int j = lower ? i : i - half, mate = lower ? i + half : i - half;
          const float c = trig[j], sn = lower ? -trig[half + j] : trig[half + j];
          qv = qv * c + to_f32(q[t * a.q_stride + mate]) * sn;
          kv = kv * c + to_f32(k[t * a.k_stride + mate]) * sn;
        }
        if (MEMORY) qv *= a.k_scale;
        else kv *= a.k_scale;
      }
      sq[i] = qv;
      sk[i] = kv;
      if (CHANNEL) {
        sa[i] = i < a.d ? expf(a.channel_decay[t * a.channel_decay_stride + (int64_t)g * a.d + i]) : 0.f;
        su[i] = i < a.d ? a.bonus[(int64_t)g * a.d + i] * kv : 0.f;
      }
    }
    for (int i = tid; i < kRows; i += 256) {
      float x = 0.f;
      if (row0 + i < a.vd) {
        x = to_f32(v[t * a.v_stride + i]);
        if (CONV) x = conv(x, (int64_t)a.v_channel + (int64_t)h * a.vd + row0 + i, pos, true);
      }
      sv[i] = x;
    }
    float decay = const_decay, scale = 1.f;
    if (a.dt) {
      scale = softplus_f32(to_f32(((const T*)a.dt)[t * a.dt_stride + h]) + bias);
      decay = expf(neg_a * scale);
    }
    float least = 0.f;
    if (MEMORY) {
      const float i = capped_gate(to_f32(((const T*)a.input_gate)[t * a.gate_stride + h]) + a.input_bias[h], a.gate_cap);
      const float f = log_sigmoid(capped_gate(to_f32(((const T*)a.forget_gate)[t * a.gate_stride + h]) + a.forget_bias[h], a.gate_cap));
      const float m_new = fmaxf(f + m, i);
      decay = expf(f + m - m_new);
      scale = expf(i - m_new);
      least = expf(-m_new);
      m = m_new;
    }
    __syncthreads();
    float kk[DPT], qq[DPT], aa[CHANNEL ? DPT : 1];
    float direct = 0.f;      // CHANNEL: this lane's part of sum u k q
#pragma unroll
    for (int p = 0; p < DPT / kPiece; ++p)
#pragma unroll
      for (int e = 0; e < kPiece; ++e) {
        kk[p * kPiece + e] = sk[piece_at(p) + e];
        qq[p * kPiece + e] = sq[piece_at(p) + e];
        if (CHANNEL) {
          aa[p * kPiece + e] = sa[piece_at(p) + e];
          direct += su[piece_at(p) + e] * qq[p * kPiece + e];
        }
      }
    float inv = 1.f;
    if (MEMORY) {
      float dot = 0.f;
#pragma unroll
      for (int e = 0; e < DPT; ++e) {
        nn[MEMORY ? e : 0] = decay * nn[MEMORY ? e : 0] + scale * kk[e];
        dot += nn[MEMORY ? e : 0] * qq[e];
      }
      inv = 1.0f / (fmaxf(fabsf(group_sum<16>(dot)), least) + kMemoryEps);
    }
#pragma unroll
    for (int r = 0; r < RPT; ++r) {
      const int row = r16 + 16 * r;
      const float x = sv[row], xs = x * scale;
      float dot = 0.f;
#pragma unroll
      for (int e = 0; e < DPT; ++e) {
        if (CHANNEL) {
          dot += s[r][e] * qq[e];
          s[r][e] = aa[CHANNEL ? e : 0] * s[r][e] + kk[e] * x;
        } else {
          s[r][e] = decay * s[r][e] + kk[e] * xs;
          dot += s[r][e] * qq[e];
        }
      }
      if (CHANNEL) dot += direct * x;
      dot = group_sum<16>(dot);
      if (ln == 0 && row0 + row < a.vd) out[t * a.out_stride + row] = from_f32<T>(MEMORY ? dot * inv : dot + skip * x);
    }
    __syncthreads();
  }
#pragma unroll
  for (int r = 0; r < RPT; ++r) {
    const int row = r16 + 16 * r;
#pragma unroll
    for (int p = 0; p < DPT / kPiece; ++p) {
      const int i = piece_at(p);
      if (row0 + row < a.vd && i < a.pitch) {
        float v[kPiece];
#pragma unroll
        for (int e = 0; e < kPiece; ++e) v[e] = s[r][p * kPiece + e];
        if (kPiece == 4) store_vec<kPiece>(state + (int64_t)row * a.pitch + i, v);
        else {
#pragma unroll
          for (int e = 0; e < kPiece; ++e) state[(int64_t)row * a.pitch + i + e] = v[e];
        }
      }
    }
  }
  if (MEMORY) {
    if (r16 == 0) {
#pragma unroll
      for (int p = 0; p < DPT / kPiece; ++p)
#pragma unroll
        for (int e = 0; e < kPiece; ++e)
          if (piece_at(p) + e < a.pitch) n_row[piece_at(p) + e] = nn[MEMORY ? p * kPiece + e : 0];
    }
    if (tid == 0) *top = m;      // behind the barriers above: everyone has read it
  }
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void short_conv_kernel(const T* __restrict__ x, int64_t x_stride, const float* __restrict__ w,
                                                         const float* __restrict__ bias, const T* __restrict__ ring,
                                                         const int32_t* __restrict__ token_seq, const int32_t* __restrict__ cu_seqlens,
                                                         const int32_t* __restrict__ starts, const int32_t* __restrict__ state_slots,
                                                         int64_t num_slots, T* __restrict__ out, int64_t tokens, int64_t channels,
                                                         int taps) {
  const int64_t pieces = channels / VEC;
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= tokens * pieces) return;
  const int64_t t = i / pieces;
  const int64_t c = (i % pieces) * VEC;
  const int b = token_seq[t];
  const int slot = state_slots[b];
  const int in_portion = (int)t - cu_seqlens[b];
  const int pos = starts[b] + in_portion;
  float acc[VEC], v[VEC], wv[VEC];
#pragma unroll
  for (int e = 0; e < VEC; ++e) acc[e] = 0.f;
  if (bias) load_vec<VEC>(bias + c, acc);
  for (int lag = 0; lag < taps; ++lag) {
    if (pos - lag < 0) break;
    if (lag <= in_portion) load_vec<VEC>(x + (t - lag) * x_stride + c, v);
    else if (slot >= 0 && slot < num_slots) load_vec<VEC>(ring + ((int64_t)slot * taps + (pos - lag) % taps) * channels + c, v);
    else break;
    load_vec<VEC>(w + (int64_t)(taps - 1 - lag) * channels + c, wv);
#pragma unroll
    for (int e = 0; e < VEC; ++e) acc[e] += wv[e] * v[e];
  }
#pragma unroll
  for (int e = 0; e < VEC; ++e) acc[e] = silu_for<T>(acc[e]);
  store_vec<VEC>(out + t * channels + c, acc);
}

// The same for the usual tap counts: a thread keeps the weights and the last TAPS inputs of eight channels in registers and
// walks kConvRun tokens, reading each input once.
constexpr int kConvRun = 16;

template <typename T, int TAPS>
__global__ __launch_bounds__(256) void short_conv_run_kernel(const T* __restrict__ x, int64_t x_stride, const float* __restrict__ w,
                                                             const float* __restrict__ bias, const T* __restrict__ ring,
                                                             const int32_t* __restrict__ token_seq, const int32_t* __restrict__ cu_seqlens,
                                                             const int32_t* __restrict__ starts, const int32_t* __restrict__ state_slots,
                                                             int64_t num_slots, T* __restrict__ out, int64_t tokens, int64_t channels) {
  const int64_t pieces = channels / 8;
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  const int64_t t0 = i / pieces * kConvRun;
  if (t0 >= tokens) return;
  const int64_t c = (i % pieces) * 8;
  const int64_t t1 = t0 + kConvRun < tokens ? t0 + kConvRun : tokens;
  float wv[TAPS][8], b[8], win[TAPS][8];       // win[l]: the input l tokens back
#pragma unroll
  for (int l = 0; l < TAPS; ++l) load_vec<8>(w + (int64_t)(TAPS - 1 - l) * channels + c, wv[l]);
#pragma unroll
  for (int e = 0; e < 8; ++e) b[e] = 0.f;
  if (bias) load_vec<8>(bias + c, b);
  // the window in front of token t: rows of the portion, the ring behind them, zeros before the start
  auto fill = [&](int64_t t, int sq) {
    const int slot = state_slots[sq], in_portion = (int)t - cu_seqlens[sq], pos = starts[sq] + in_portion;
#pragma unroll
    for (int l = 1; l < TAPS; ++l) {
#pragma unroll
      for (int e = 0; e < 8; ++e) win[l - 1][e] = 0.f;
      if (pos - l >= 0) {
        if (l <= in_portion) load_vec<8>(x + (t - l) * x_stride + c, win[l - 1]);
        else if (slot >= 0 && slot < num_slots) load_vec<8>(ring + ((int64_t)slot * TAPS + (pos - l) % TAPS) * channels + c, win[l - 1]);
      }
    }
  };
  auto next = [&](int64_t t, const float (&in)[8]) {
#pragma unroll
    for (int l = TAPS - 1; l > 0; --l)
#pragma unroll
      for (int e = 0; e < 8; ++e) win[l][e] = win[l - 1][e];
    float acc[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      win[0][e] = in[e];
      acc[e] = b[e];
#pragma unroll
      for (int l = 0; l < TAPS; ++l) acc[e] += wv[l][e] * win[l][e];
      acc[e] = silu_for<T>(acc[e]);
    }
    store_vec<8>(out + t * channels + c, acc);
  };
  int seq = token_seq[t0];
  fill(t0, seq);
  if (t1 - t0 == kConvRun && token_seq[t1 - 1] == seq) {      // one sequence throughout: inputs four tokens ahead
#pragma unroll
    for (int j = 0; j < kConvRun; j += 4) {
      float in[4][8];
#pragma unroll
      for (int i = 0; i < 4; ++i) load_vec<8>(x + (t0 + j + i) * x_stride + c, in[i]);
#pragma unroll
      for (int i = 0; i < 4; ++i) next(t0 + j + i, in[i]);
    }
    return;
  }
  for (int64_t t = t0; t < t1; ++t) {
    const int sq = token_seq[t];
    if (sq != seq) {
      seq = sq;
      fill(t, sq);
    }
    float in[8];
    load_vec<8>(x + t * x_stride + c, in);
    next(t, in);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void short_conv_update_kernel(const T* __restrict__ x, int64_t x_stride, T* __restrict__ ring,
                                                                const int32_t* __restrict__ cu_seqlens, const int32_t* __restrict__ starts,
                                                                const int32_t* __restrict__ state_slots, int64_t num_slots,
                                                                int64_t channels, int taps) {
  const int b = blockIdx.y;
  const int64_t c = (int64_t)blockIdx.x * 256 + threadIdx.x;
  const int slot = state_slots[b];
  if (c >= channels || slot < 0 || slot >= num_slots) return;
  const int t0 = cu_seqlens[b], n = cu_seqlens[b + 1] - t0, start = starts[b];
  for (int j = n > taps - 1 ? n - (taps - 1) : 0; j < n; ++j)
    ring[((int64_t)slot * taps + (start + j) % taps) * channels + c] = x[(int64_t)(t0 + j) * x_stride + c];
}

template <typename T, int DPT, RecurrenceKind KIND>
static void launch_recurrence_kind(const RecurrenceArgs& a, int64_t batch, hipStream_t s) {
#define MOPS_REC(R)                                                                                                      \
  hipLaunchKernelGGL((decayed_recurrence_kernel<T, DPT, R, KIND>), dim3((unsigned)(batch * a.heads * ((a.vd + 16 * (R) - 1) / (16 * (R))))), \
                     dim3(256), 0, s, a)
  if (a.vd <= 16) MOPS_REC(1);
  else if (a.vd <= 32) MOPS_REC(2);
  else MOPS_REC(4);
#undef MOPS_REC
}

template <typename T, int DPT>
static void launch_recurrence_rows(const RecurrenceArgs& a, int64_t batch, bool conv, hipStream_t s) {
  if (a.channel_decay) launch_recurrence_kind<T, DPT, kPerChannel>(a, batch, s);
  else if (a.input_gate) launch_recurrence_kind<T, DPT, kMemory>(a, batch, s);
  else if (conv) launch_recurrence_kind<T, DPT, kConvolved>(a, batch, s);
  else launch_recurrence_kind<T, DPT, kPlain>(a, batch, s);
}

template <typename T>
static int launch_recurrence(const RecurrenceArgs& a, int64_t batch, bool conv, hipStream_t s) {
  if (a.d <= 32) launch_recurrence_rows<T, 2>(a, batch, conv, s);
  else if (a.d <= 64) launch_recurrence_rows<T, 4>(a, batch, conv, s);
  else if (a.d <= 128) launch_recurrence_rows<T, 8>(a, batch, conv, s);
  else if (a.d <= 256) launch_recurrence_rows<T, 16>(a, batch, conv, s);
  else if (a.d <= 512) launch_recurrence_rows<T, 32>(a, batch, conv, s);
  else return MOPS_HIP_EUNSUPPORTED;
  return finish_launch();
}

}  // namespace mops

extern "C" int64_t mops_hip_matrix_memory_copies(int64_t vd) { return vd <= 0 ? MOPS_HIP_EINVAL : (vd + 63) / 64; }

extern "C" int64_t mops_hip_recurrence_state_pitch(int64_t d) { return d <= 0 ? MOPS_HIP_EINVAL : (d + 3) / 4 * 4; }

extern "C" int mops_hip_decayed_recurrence(const mops_hip_recurrence* r, void* stream) {
  using namespace mops;
  if (!r || !known_dtype(r->dtype) || r->batch < 0) return MOPS_HIP_EINVAL;
  if (r->batch == 0) return MOPS_HIP_OK;
  if (!r->q || !r->k || !r->v || !r->out || !r->state || !r->state_slots || !r->starts) return MOPS_HIP_EINVAL;
  if (r->heads <= 0 || r->groups <= 0 || r->heads % r->groups || r->d <= 0 || r->vd <= 0 || r->num_slots <= 0) return MOPS_HIP_EINVAL;
  if (r->d > 512 || r->heads > 65536 || r->vd > 65536) return MOPS_HIP_EUNSUPPORTED;
  if (r->q_stride < r->groups * r->d || r->k_stride < r->groups * r->d || r->v_stride < r->heads * r->vd ||
      r->out_stride < r->heads * r->vd)
    return MOPS_HIP_EINVAL;
  if ((r->decay != nullptr) + (r->dt != nullptr) + (r->channel_decay != nullptr) + (r->input_gate != nullptr) != 1) return MOPS_HIP_EINVAL;      // one source of the decay
  if (r->input_gate && (!r->forget_gate || !r->input_bias || !r->forget_bias || !r->top || !(r->gate_cap > 0.f) || r->gate_stride < r->heads || r->skip ||
                        r->conv_weight))
    return MOPS_HIP_EINVAL;
  if (r->channel_decay && (!r->bonus || r->groups != r->heads || r->skip || r->conv_weight || r->channel_decay_stride < r->heads * r->d)) return MOPS_HIP_EINVAL;
  if (r->dt && (!r->dt_bias || !r->neg_a || r->dt_stride < r->heads)) return MOPS_HIP_EINVAL;
  if (r->rot < 0 || (r->rot & 1) || r->rot > r->d || (r->rot && (!r->cos_sin || r->max_positions <= 0))) return MOPS_HIP_EINVAL;
  const bool conv = r->conv_weight != nullptr;
  if (conv && (r->cu_seqlens || r->rot || !r->conv_bias || !r->conv_ring || r->taps <= 0 || r->channels <= 0 ||
               r->q_channel < 0 || r->k_channel < 0 || r->v_channel < 0 || r->q_channel + r->groups * r->d > r->channels ||
               r->k_channel + r->groups * r->d > r->channels || r->v_channel + r->heads * r->vd > r->channels))
    return MOPS_HIP_EINVAL;
  if (!aligned16(r->state)) return MOPS_HIP_EALIGN;
  if (r->batch * r->heads * ((r->vd + 15) / 16) > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  RecurrenceArgs a;
  a.q = r->q; a.k = r->k; a.v = r->v;
  a.q_stride = r->q_stride; a.k_stride = r->k_stride; a.v_stride = r->v_stride;
  a.out = r->out; a.out_stride = r->out_stride;
  a.state = r->state; a.num_slots = r->num_slots;
  a.state_slots = r->state_slots; a.cu_seqlens = r->cu_seqlens; a.starts = r->starts;
  a.heads = (int)r->heads; a.groups = (int)r->groups; a.d = (int)r->d; a.vd = (int)r->vd;
  a.pitch = (int)mops_hip_recurrence_state_pitch(r->d);
  a.decay = r->decay; a.dt = r->dt; a.dt_stride = r->dt_stride; a.dt_bias = r->dt_bias; a.neg_a = r->neg_a; a.skip = r->skip;
  a.channel_decay = r->channel_decay; a.channel_decay_stride = r->channel_decay_stride; a.bonus = r->bonus;
  a.input_gate = r->input_gate; a.forget_gate = r->forget_gate; a.gate_stride = r->gate_stride;
  a.input_bias = r->input_bias; a.forget_bias = r->forget_bias; a.gate_cap = r->gate_cap;
  a.top = r->top; a.copies = r->input_gate ? (int)mops_hip_matrix_memory_copies(r->vd) : 0;
  a.cos_sin = r->cos_sin; a.rot = (int)r->rot; a.max_positions = r->max_positions; a.k_scale = r->k_scale;
  a.conv_w = r->conv_weight; a.conv_b = r->conv_bias; a.ring = r->conv_ring; a.taps = (int)r->taps; a.channels = r->channels;
  a.q_channel = (int)r->q_channel; a.k_channel = (int)r->k_channel; a.v_channel = (int)r->v_channel;
  return r->dtype == MOPS_HIP_BF16 ? launch_recurrence<bf16_t>(a, r->batch, conv, (hipStream_t)stream)
                                   : launch_recurrence<float>(a, r->batch, conv, (hipStream_t)stream);
}

extern "C" int mops_hip_short_conv(const void* x, int64_t x_row_stride, const float* weight, const float* bias, const void* ring,
                                   int64_t num_slots, const int32_t* token_seq, const int32_t* cu_seqlens, const int32_t* starts,
                                   const int32_t* state_slots, void* out, int dtype, int64_t tokens, int64_t channels, int64_t taps,
                                   void* stream) {
  using namespace mops;
  if (!known_dtype(dtype) || tokens < 0 || channels <= 0 || taps <= 0 || taps > 1024 || num_slots <= 0) return MOPS_HIP_EINVAL;
  if (tokens == 0) return MOPS_HIP_OK;
  if (!x || !weight || !ring || !token_seq || !cu_seqlens || !starts || !state_slots || !out || x_row_stride < channels)
    return MOPS_HIP_EINVAL;
  const bool vec = channels % 8 == 0 && x_row_stride % 8 == 0 && aligned16(x) && aligned16(weight) && (!bias || aligned16(bias)) && aligned16(ring) && aligned16(out);
  const int64_t wgs = (tokens * (channels / (vec ? 8 : 1)) + 255) / 256;
  if (wgs > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  hipStream_t s = (hipStream_t)stream;
  if (vec && tokens >= 256 && taps >= 2 && taps <= 4) {
    const dim3 grid((unsigned)(((tokens + kConvRun - 1) / kConvRun * (channels / 8) + 255) / 256));
#define MOPS_CONV_RUN(T, N) hipLaunchKernelGGL((short_conv_run_kernel<T, N>), grid, dim3(256), 0, s, (const T*)x, x_row_stride, weight, bias, \
                            (const T*)ring, token_seq, cu_seqlens, starts, state_slots, num_slots, (T*)out, tokens, channels)
#define MOPS_CONV_TAPS(T) do { if (taps == 2) MOPS_CONV_RUN(T, 2); else if (taps == 3) MOPS_CONV_RUN(T, 3); else MOPS_CONV_RUN(T, 4); } while (0)
    if (dtype == MOPS_HIP_BF16) MOPS_CONV_TAPS(bf16_t);
    else MOPS_CONV_TAPS(float);
#undef MOPS_CONV_TAPS
#undef MOPS_CONV_RUN
    return finish_launch();
  }
#define MOPS_CONV(T, V) hipLaunchKernelGGL((short_conv_kernel<T, V>), dim3((unsigned)wgs), dim3(256), 0, s, (const T*)x, x_row_stride, weight, \
                        bias, (const T*)ring, token_seq, cu_seqlens, starts, state_slots, num_slots, (T*)out, tokens, channels, (int)taps)
  if (dtype == MOPS_HIP_BF16) { if (vec) MOPS_CONV(bf16_t, 8); else MOPS_CONV(bf16_t, 1); }
  else { if (vec) MOPS_CONV(float, 8); else MOPS_CONV(float, 1); }
#undef MOPS_CONV
  return finish_launch();
}

extern "C" int mops_hip_short_conv_update(const void* x, int64_t x_row_stride, void* ring, int64_t num_slots, const int32_t* cu_seqlens,
                                          const int32_t* starts, const int32_t* state_slots, int dtype, int64_t batch, int64_t channels,
                                          int64_t taps, void* stream) {
  using namespace mops;
  if (!known_dtype(dtype) || batch < 0 || channels <= 0 || taps <= 0 || taps > 1024 || num_slots <= 0) return MOPS_HIP_EINVAL;
  if (batch == 0) return MOPS_HIP_OK;
  if (!x || !ring || !cu_seqlens || !starts || !state_slots || x_row_stride < channels) return MOPS_HIP_EINVAL;
  if (batch > 65535) return MOPS_HIP_EUNSUPPORTED;
  const dim3 grid((unsigned)((channels + 255) / 256), (unsigned)batch);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MOPS_HIP_BF16)
    hipLaunchKernelGGL((short_conv_update_kernel<bf16_t>), grid, dim3(256), 0, s, (const bf16_t*)x, x_row_stride, (bf16_t*)ring, cu_seqlens,
                       starts, state_slots, num_slots, channels, (int)taps);
  else
    hipLaunchKernelGGL((short_conv_update_kernel<float>), grid, dim3(256), 0, s, (const float*)x, x_row_stride, (float*)ring, cu_seqlens, starts,
                       state_slots, num_slots, channels, (int)taps);
  return finish_launch();
}
