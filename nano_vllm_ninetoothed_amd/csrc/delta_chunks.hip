// The gated delta rule (delta_rule.hip) for portions of many tokens, 16 tokens at a time on the matrix cores (bf16 in, float32
// accumulation and state).  With L_t = log2 of the product of the decays of a chunk up to token t (per channel), b_t the write strength
// and S the state in front of the chunk, the writes u_t of a chunk solve a triangular system:
//
//   u_t = b_t (v_t - S^T (2^{L_t} k_t) - sum_{j<t} A[t, j] u_j),   A[t, j] = sum_d k_t k_j 2^{L_t - L_j}
//   o_t = S^T (2^{L_t} q_t) + sum_{j<=t} P[t, j] u_j,              P[t, j] = sum_d q_t k_j 2^{L_t - L_j}
//   S  <- 2^{L_15} S + sum_j (2^{L_15 - L_j} k_j) u_j^T
//
// With T = (1 + diag(b) A)^-1 diag(b) (1 + a strictly lower triangular matrix, inverted by substitution) the writes are
// U = T V - W S, W = T (2^L k): everything but the products with S is known without S.  Two kernels:
//
//   delta_prepare_kernel   a wave per (chunk, head), all chunks in parallel: unit vectors, cumulative decays, A, P, T and W, left in memory
//                          as the operands of the second kernel's products, lane by lane, so that it reads 16 bytes per lane in a row
//   delta_scan_kernel      a wave per (sequence, head, 16 value columns) walks the chunks with S [d x 16] in its accumulators:
//                          U = T V - W S, O^T = S^T q + U^T P^T, S <- 2^{L_15} S + k^T U; the waves of a workgroup share the operands
//
// A sequence is one segment when sequences and heads fill the chip.  Otherwise it is cut, and three launches walk the segments side by side:
//   states from zero   U = T V - W S without outputs, and beside the value columns d more with V = 0 that start from the identity: what the
//                      segment makes of the state in front of it is S <- M S + C
//   delta_join_kernel  S at the start of every segment, one after the other, and the last state into the sequence's slot
//   outputs            delta_scan_kernel from these
//
// A and P come apart into one factor per token on either side of a reference as in channel_chunks.hip: L_7 where t >= 8 > j, else the
// middle of the half chunk both lie in (a decay below 2^-28 counts as 2^-28).  What is kept in 32 bits enters a product as the sum of two
// bf16 numbers; where a product is 16 deep the two halves of the 32 deep instruction hold them.
// A lane holds channels 32 s + 4 jj + 0..3 and 16 further on of step s in the first kernel, which is the order in which the accumulators
// of S are an operand of the second.
#include "mfma_tiles.h"

namespace mops {

constexpr int kDTokens = 16;
constexpr float kLeastLog2Keep = -28.f;
constexpr int kPieceBytes = 1024;      // an operand of a wave: 16 bytes per lane

struct DeltaChunkArgs {
  mops_hip_delta a;
  const int32_t* chunks;        // [n][2]: first token, tokens
  const int32_t* segments;      // [n][4]: sequence, first token, one past the last, first chunk
  const int32_t* seq_segments;  // [batch + 1]
  int num_chunks, num_segments, pitch;
  unsigned char* operands;      // per (chunk, head): Q hi, Q lo [d / 32], P, W hi, W lo, K [d / 16], T as pieces, then 2^{L_15} float [d]
  float* seg_state;             // [segments][heads][vd][pitch]: C, then the state at the start; nullptr: one segment per sequence
  unsigned char* seg_map;       // [segments][heads]: M hi, M lo as pieces [d / 16][d / 32]
  bool vec;
};

template <int DP>
struct DeltaShape {
  static constexpr int kSteps = DP / 32, kTiles = DP / 16;
  static constexpr int kQ = 0, kP = 2 * kSteps, kW = kP + 1, kK = kW + 2 * kSteps, kT = kK + kTiles, kPieces = kT + 1;
  static constexpr int64_t kBytes = kPieces * kPieceBytes + DP * 4;
  static constexpr int64_t kMapBytes = 2 * kTiles * kSteps * kPieceBytes;
  // the operands that a pass reads are in one run
  static constexpr int from(bool states) { return states ? kW * kPieceBytes : 0; }
};

template <int N>
__device__ __forceinline__ float row_up(float v) {       // the lane N places in front inside the row of 16; 0 where there is none
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x110 | N, 0xf, 0xf, true));
}
template <int N>
__device__ __forceinline__ float row_take(float v) {     // lane N of the row of 16
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x150 | N, 0xf, 0xf, true));
}
__device__ __forceinline__ void wave_sync() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}
// Four values as hi (words 0, 1) and lo (words 2, 3).
__device__ __forceinline__ u32x4 split4(const float (&v)[4]) {
  u32x4 w;
  w[0] = pack_bf16x2(v[0], v[1]);
  w[1] = pack_bf16x2(v[2], v[3]);
  w[2] = pack_bf16x2(v[0] - bf16lo_to_f32(w[0]), v[1] - bf16hi_to_f32(w[0]));
  w[3] = pack_bf16x2(v[2] - bf16lo_to_f32(w[1]), v[3] - bf16hi_to_f32(w[1]));
  return w;
}
__device__ __forceinline__ bf16x8 as_operand(u32x4 w) { return __builtin_bit_cast(bf16x8, w); }
__device__ __forceinline__ bf16x8 high_twice(u32x4 w) { return as_operand(u32x4{w[0], w[1], w[0], w[1]}); }
__device__ __forceinline__ bf16x8 low_once(u32x4 w) { return as_operand(u32x4{w[2], w[3], 0u, 0u}); }

template <int DP, int WAVES>
__global__ __launch_bounds__(64 * WAVES) void delta_prepare_kernel(const DeltaChunkArgs p) {
  using Sh = DeltaShape<DP>;
  constexpr int kS = Sh::kSteps, kPitch = DP + 8;
  __shared__ __align__(16) uint16_t tiles[WAVES][2][kDTokens * kPitch];
  const mops_hip_delta& a = p.a;
  const int heads = (int)a.heads, d = (int)a.d;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, n16 = lane & 15, jj = lane >> 4;
  const int64_t item = (int64_t)blockIdx.x * WAVES + wave;
  if (item >= (int64_t)p.num_chunks * heads) return;      // no workgroup barriers below
  const int h = (int)(item % heads), chunk = (int)(item / heads);
  const int first = p.chunks[2 * chunk], n = p.chunks[2 * chunk + 1];
  const bool in = n16 < n;
  const int64_t t = first + (in ? n16 : n - 1);
  const int g = h / (heads / (int)a.groups);
  const uint16_t *qp = (const uint16_t*)a.q + t * a.q_stride + (int64_t)g * d, *kp = (const uint16_t*)a.k + t * a.k_stride + (int64_t)g * d;
  const float* lp = a.log_decay + t * a.log_decay_stride + (int64_t)h * d;
  float beta = sigmoid_for<float>(bf16lo_to_f32(((const uint16_t*)a.beta)[t * a.beta_stride + h]));
  if (!in) beta = 0.f;

  float q[kS][8], k[kS][8], L[kS][8];
#pragma unroll
  for (int s = 0; s < kS; ++s)
#pragma unroll
    for (int half = 0; half < 2; ++half) {
      const int c = 32 * s + 16 * half + 4 * jj;
      if (p.vec) {
        const int cc = c < d ? c : 0;
        const u32x2 x = *reinterpret_cast<const u32x2*>(qp + cc), y = *reinterpret_cast<const u32x2*>(kp + cc);
        const f32x4 z = *reinterpret_cast<const f32x4*>(lp + cc);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          q[s][4 * half + e] = e & 1 ? bf16hi_to_f32(x[e >> 1]) : bf16lo_to_f32(x[e >> 1]);
          k[s][4 * half + e] = e & 1 ? bf16hi_to_f32(y[e >> 1]) : bf16lo_to_f32(y[e >> 1]);
          L[s][4 * half + e] = z[e];
        }
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int cc = c + e < d ? c + e : 0;
          q[s][4 * half + e] = bf16lo_to_f32(qp[cc]);
          k[s][4 * half + e] = bf16lo_to_f32(kp[cc]);
          L[s][4 * half + e] = lp[cc];
        }
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const bool ok = in && c + e < d;
        const int i = 4 * half + e;
        q[s][i] = ok ? q[s][i] : 0.f;
        k[s][i] = ok ? k[s][i] : 0.f;
        L[s][i] = ok ? fmaxf(L[s][i] * 1.4426950408889634f, kLeastLog2Keep) : 0.f;
      }
    }
  float qq = 0.f, kk = 0.f;
#pragma unroll
  for (int s = 0; s < kS; ++s)
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      qq += q[s][e] * q[s][e];
      kk += k[s][e] * k[s][e];
      float x = L[s][e];
      x += row_up<1>(x);
      x += row_up<2>(x);
      x += row_up<4>(x);
      x += row_up<8>(x);
      L[s][e] = x;
    }
  qq += __shfl_xor(qq, 16, kWave);
  kk += __shfl_xor(kk, 16, kWave);
  qq += __shfl_xor(qq, 32, kWave);
  kk += __shfl_xor(kk, 32, kWave);
  const float rq = a.q_scale / sqrtf(qq + a.unit_eps), rk = 1.0f / sqrtf(kk + a.unit_eps);

  unsigned char* const dst = p.operands + item * Sh::kBytes;
  auto put = [&](int piece, u32x4 w) { store16(dst + piece * kPieceBytes + lane * 16, w); };
  float* const decay = reinterpret_cast<float*>(dst + Sh::kPieces * kPieceBytes);
  uint16_t* const hi_tile = tiles[wave][0];
  uint16_t* const lo_tile = tiles[wave][1];
  auto row_store = [&](int s, const float (&v)[8]) {      // a step's eight values of token n16 into the tiles
#pragma unroll
    for (int half = 0; half < 2; ++half) {
      const float x[4] = {v[4 * half], v[4 * half + 1], v[4 * half + 2], v[4 * half + 3]};
      const u32x4 w = split4(x);
      const int at = n16 * kPitch + 32 * s + 16 * half + 4 * jj;
      *reinterpret_cast<u32x2*>(hi_tile + at) = u32x2{w[0], w[1]};
      *reinterpret_cast<u32x2*>(lo_tile + at) = u32x2{w[2], w[3]};
    }
  };

  // ---- A and P: [j = 4 jj + e][t = n16], inside the halves of the chunk and across
  f32x4 a_in = {0.f, 0.f, 0.f, 0.f}, p_in = a_in, a_over = a_in, p_over = a_in;
#pragma unroll
  for (int s = 0; s < kS; ++s) {
    float kt[8], qt[8], kj[8], kb[8], qb[8], grown[8], qf[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      q[s][e] *= rq;
      k[s][e] *= rk;
      const float l = L[s][e], m3 = row_take<3>(l), m7 = row_take<7>(l), m11 = row_take<11>(l), mid = n16 < 8 ? m3 : m11;
      const float up = __builtin_amdgcn_exp2f(l - mid), whole = __builtin_amdgcn_exp2f(l);
      kt[e] = k[s][e] * up;
      qt[e] = q[s][e] * up;
      kj[e] = k[s][e] * __builtin_amdgcn_exp2f(mid - l);
      const float over = __builtin_amdgcn_exp2f(n16 < 8 ? m7 - l : l - m7);
      kb[e] = k[s][e] * over;
      qb[e] = n16 < 8 ? 0.f : q[s][e] * over;
      grown[e] = k[s][e] * whole;
      qf[e] = q[s][e] * whole;
    }
    bf16x8 kth, ktl, qth, qtl, kjh, kjl, kbh, kbl, qbh, qbl, qfh, qfl;
    split8(kt, kth, ktl);
    split8(qt, qth, qtl);
    split8(kj, kjh, kjl);
    split8(kb, kbh, kbl);
    split8(qb, qbh, qbl);
    split8(qf, qfh, qfl);
    a_in = mfma16(kjh, kth, a_in);
    p_in = mfma16(kjh, qth, p_in);
    a_over = mfma16(kbh, kbh, a_over);
    p_over = mfma16(kbh, qbh, p_over);
    a_in = mfma16(kjh, ktl, a_in);
    p_in = mfma16(kjh, qtl, p_in);
    a_over = mfma16(kbh, kbl, a_over);
    p_over = mfma16(kbh, qbl, p_over);
    a_in = mfma16(kjl, kth, a_in);
    p_in = mfma16(kjl, qth, p_in);
    a_over = mfma16(kbl, kbh, a_over);
    p_over = mfma16(kbl, qbh, p_over);
    put(Sh::kQ + s, __builtin_bit_cast(u32x4, qfh));
    put(Sh::kQ + kS + s, __builtin_bit_cast(u32x4, qfl));
    row_store(s, grown);
  }
  float below[4], weight[4], beta_j[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const int j = 4 * jj + e;
    const bool over = n16 >= 8 && j < 8;
    below[e] = j < n16 ? beta * (over ? a_over[e] : a_in[e]) : 0.f;
    weight[e] = j <= n16 ? (over ? p_over[e] : p_in[e]) : 0.f;
    beta_j[e] = __shfl(beta, j, kWave);
  }
  put(Sh::kP, split4(weight));

  // ---- T: lane = row t, from the last column to the first; x[j] = [t == j] - sum_{i > j} x[i] below[i, j]
  float x[kDTokens];
#pragma unroll
  for (int j = kDTokens - 1; j >= 0; --j) {
    float acc = n16 == j ? 1.f : 0.f;
#pragma unroll
    for (int i = j + 1; i < kDTokens; ++i)
      acc -= x[i] * __int_as_float(__builtin_amdgcn_readlane(__float_as_int(below[j & 3]), 16 * (j >> 2) + i));
    x[j] = acc;
  }
  float tb[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) tb[e] = (jj < 2 ? (jj == 0 ? x[e] : x[4 + e]) : (jj == 2 ? x[8 + e] : x[12 + e])) * beta_j[e];
  const u32x4 tw = split4(tb);
  put(Sh::kT, tw);

  // ---- -W^T [d, t] = -(2^L k)^T T^T, in the order of an operand
  wave_sync();
  const bf16x8 t_high = high_twice(tw), t_low = low_once(tw);
#pragma unroll
  for (int s = 0; s < kS; ++s) {
    float w[8];
#pragma unroll
    for (int half = 0; half < 2; ++half) {
      const s16x4 kh = tile_block_columns(hi_tile, kPitch, 4 * jj, 32 * s + 16 * half, lane), kl = tile_block_columns(lo_tile, kPitch, 4 * jj, 32 * s + 16 * half, lane);
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
      acc = mfma16(__builtin_bit_cast(bf16x8, join(kh, kl)), t_high, acc);
      acc = mfma16(__builtin_bit_cast(bf16x8, join(kh, kh)), t_low, acc);
#pragma unroll
      for (int e = 0; e < 4; ++e) w[4 * half + e] = -acc[e];
    }
    bf16x8 hi, lo;
    split8(w, hi, lo);
    put(Sh::kW + s, __builtin_bit_cast(u32x4, hi));
    put(Sh::kW + kS + s, __builtin_bit_cast(u32x4, lo));
  }
  wave_sync();
  // ---- 2^{L_15 - L} k, columns of it
#pragma unroll
  for (int s = 0; s < kS; ++s) {
    float w[8], end[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      end[e] = row_take<15>(L[s][e]);
      w[e] = k[s][e] * __builtin_amdgcn_exp2f(end[e] - L[s][e]);
    }
    row_store(s, w);
    if (n16 == 0) {
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        f32x4 v;
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = __builtin_amdgcn_exp2f(end[4 * half + e]);
        *reinterpret_cast<f32x4*>(decay + 32 * s + 16 * half + 4 * jj) = v;
      }
    }
  }
  wave_sync();
#pragma unroll
  for (int i = 0; i < Sh::kTiles; ++i)
    put(Sh::kK + i, __builtin_bit_cast(u32x4, join(tile_block_columns(hi_tile, kPitch, 4 * jj, 16 * i, lane), tile_block_columns(lo_tile, kPitch, 4 * jj, 16 * i, lane))));
}

// WAVES waves of 16 value columns each.  The operands of a chunk go through LDS, two buffers; two more chunks are on their way in
// registers, so that a load has two chunks' time to come back.
template <int DP, int WAVES, bool STATES>
__global__ __launch_bounds__(64 * WAVES) void delta_scan_kernel(const DeltaChunkArgs p) {
  using Sh = DeltaShape<DP>;
  constexpr int kS = Sh::kSteps, kI = Sh::kTiles, kThreads = 64 * WAVES, kFrom = Sh::from(STATES);
  constexpr int kBuffer = (int)Sh::kBytes - kFrom, kLoads16 = kBuffer / 16, kLoads = (kLoads16 + kThreads - 1) / kThreads;
  extern __shared__ __align__(16) unsigned char smem[];
  const mops_hip_delta& a = p.a;
  const int heads = (int)a.heads, vd = (int)a.vd, value_columns = (vd + 15) / 16 * 16;
  const int columns = value_columns + (STATES ? ((int)a.d + 15) / 16 * 16 : 0), blocks = (columns + 16 * WAVES - 1) / (16 * WAVES);
  // each XCD a contiguous run of items, so that the workgroups of a head share an L2
  const int total = p.num_segments * heads * blocks, per_xcd = (total + 7) / 8;
  const int item = (blockIdx.x % 8) * per_xcd + blockIdx.x / 8;
  if ((int)blockIdx.x / 8 >= per_xcd || item >= total) return;
  const int h = item / blocks % heads, seg = item / (blocks * heads);
  const int tid = threadIdx.x, lane = tid & 63, n16 = lane & 15, jj = lane >> 4;
  const int v0 = item % blocks * 16 * WAVES + (tid >> 6) * 16;
  const int b = p.segments[4 * seg], t_begin = p.segments[4 * seg + 1], t_end = p.segments[4 * seg + 2], first_chunk = p.segments[4 * seg + 3];
  const int slot = a.state_slots[b];
  if (slot < 0 || slot >= a.num_slots || t_end <= t_begin) return;
  const bool active = v0 < columns, v_ok = v0 + n16 < vd, maps = STATES && v0 >= value_columns;      // maps: columns of M
  const int v = v_ok ? v0 + n16 : vd - 1;
  float* const state = (p.seg_state ? p.seg_state + ((int64_t)seg * heads + h) * vd * p.pitch : a.state + ((int64_t)slot * heads + h) * vd * p.pitch) +
                       (int64_t)v * p.pitch;
  // S: tile i, element e = row d = 16 i + 4 jj + e, column v0 + n16
  f32x4 st[kI];
  const bool load_state = !STATES && (p.seg_state || a.starts[b] > 0);
#pragma unroll
  for (int i = 0; i < kI; ++i) {
    const int d = 16 * i + 4 * jj;
    const bool ok = load_state && d < p.pitch;
    const f32x4 w = *reinterpret_cast<const f32x4*>(state + (ok ? d : 0));
#pragma unroll
    for (int e = 0; e < 4; ++e) st[i][e] = ok ? w[e] : (maps && d + e == v0 - value_columns + n16 ? 1.f : 0.f);
  }
  const uint16_t* const vp = (const uint16_t*)a.v + (int64_t)h * vd + v;
  uint16_t* const op = (uint16_t*)a.out + (int64_t)h * vd + v0 + 4 * jj;
  const int n_chunks = (t_end - t_begin + kDTokens - 1) / kDTokens;
  const unsigned char* const src = p.operands + ((int64_t)first_chunk * heads + h) * Sh::kBytes + kFrom;
  const int64_t step = heads * Sh::kBytes;

  // a chunk on its way: this thread's pieces of the operands, and its wave's values
  struct Flight {
    u32x4 w[kLoads];
    uint32_t v[4];
  } even, odd;
  auto fetch = [&](Flight& f, int chunk) {
    chunk = chunk < n_chunks ? chunk : n_chunks - 1;
    const unsigned char* from = src + chunk * step;
#pragma unroll
    for (int i = 0; i < kLoads; ++i) {
      const int at = i * kThreads + tid;
      f.w[i] = load16(from + 16 * (at < kLoads16 ? at : 0));
    }
    const int t0 = t_begin + chunk * kDTokens + 4 * jj;
#pragma unroll
    for (int e = 0; e < 4; ++e) f.v[e] = vp[(int64_t)(t0 + e < t_end ? t0 + e : t_end - 1) * a.v_stride];
  };
  auto file = [&](const Flight& f, int buffer) {
#pragma unroll
    for (int i = 0; i < kLoads; ++i) {
      const int at = i * kThreads + tid;
      if ((i + 1) * kThreads <= kLoads16 || at < kLoads16) store16(smem + buffer * kBuffer + 16 * at, f.w[i]);
    }
  };
  u32x2 vw, vw_next;
  auto values = [&](const Flight& f) { return maps ? u32x2{0u, 0u} : u32x2{f.v[0] | f.v[1] << 16, f.v[2] | f.v[3] << 16}; };
  auto run = [&](int chunk, int buffer) {
    const unsigned char* const ops = smem + buffer * kBuffer - kFrom;
    auto piece = [&](int i) { return as_operand(load16(ops + i * kPieceBytes + lane * 16)); };
    f32x4 u = {0.f, 0.f, 0.f, 0.f}, u2 = u, o = u, o2 = u;
    u = mfma16(piece(Sh::kT), as_operand(u32x4{vw[0], vw[1], vw[0], vw[1]}), u);
#pragma unroll
    for (int s = 0; s < kS; ++s) {
      float x[8];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        x[e] = st[2 * s][e];
        x[4 + e] = st[2 * s + 1][e];
      }
      bf16x8 hi, lo;
      split8(x, hi, lo);
      const bf16x8 wh = piece(Sh::kW + s), wl = piece(Sh::kW + kS + s);
      u = mfma16(wh, hi, u);
      u2 = mfma16(wh, lo, u2);
      if (!STATES) {
        const bf16x8 qh = piece(Sh::kQ + s), ql = piece(Sh::kQ + kS + s);
        o = mfma16(hi, qh, o);
        o2 = mfma16(hi, ql, o2);
        o = mfma16(lo, qh, o);
      }
      u = mfma16(wl, hi, u);
    }
    float uu[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) uu[e] = u[e] + u2[e];
    const u32x4 uw = split4(uu);
    const bf16x8 u_high = high_twice(uw), u_low = low_once(uw);
#pragma unroll
    for (int i = 0; i < kI; ++i) {
      const f32x4 keep = *reinterpret_cast<const f32x4*>(ops + Sh::kPieces * kPieceBytes + (16 * i + 4 * jj) * 4);
      const bf16x8 k = piece(Sh::kK + i);
#pragma unroll
      for (int e = 0; e < 4; ++e) st[i][e] *= keep[e];
      st[i] = mfma16(k, u_high, st[i]);
      st[i] = mfma16(k, u_low, st[i]);
    }
    if (STATES) return;
    const bf16x8 weights = piece(Sh::kP);
    o = mfma16(u_high, weights, o);
    o2 = mfma16(u_low, weights, o2);
    const int t = t_begin + chunk * kDTokens + n16;
    if (t < t_end) {
      uint16_t* const row = op + (int64_t)t * a.out_stride;
      const u32x2 w = {pack_bf16x2(o[0] + o2[0], o[1] + o2[1]), pack_bf16x2(o[2] + o2[2], o[3] + o2[3])};
      if (p.vec && v0 + 4 * jj < vd) {
        *reinterpret_cast<u32x2*>(row) = w;
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (v0 + 4 * jj + e < vd) row[e] = (uint16_t)(w[e >> 1] >> (16 * (e & 1)));
      }
    }
  };
  // one barrier per chunk: the chunk's buffer is filled, and everybody is done with the other one.  Only LDS is waited for.
  auto turn = [&](Flight& f, int chunk) {
    vw = vw_next;
    asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
    if (chunk + 1 < n_chunks) {
      file(f, (chunk + 1) & 1);
      vw_next = values(f);
      fetch(f, chunk + 3);
    }
    if (active) run(chunk, chunk & 1);
  };
  fetch(even, 0);
  fetch(odd, 1);
  file(even, 0);
  vw_next = values(even);
  fetch(even, 2);
  for (int chunk = 0; chunk < n_chunks; chunk += 2) {
    turn(odd, chunk);
    if (chunk + 1 < n_chunks) turn(even, chunk + 1);
  }
  if (maps) {      // rows of M as operands: this wave's sixteen columns are half of a step, turned in the LDS that nobody reads any more
    __syncthreads();
    if (!active) return;
    uint16_t* const hi_tile = reinterpret_cast<uint16_t*>(smem) + (tid >> 6) * 2 * 16 * 24;      // [column][16 rows], pitch 24
    uint16_t* const lo_tile = hi_tile + 16 * 24;
    unsigned char* const dst = p.seg_map + ((int64_t)seg * heads + h) * Sh::kMapBytes;
    const int m0 = v0 - value_columns, s = m0 / 32, half = m0 / 16 & 1;
#pragma unroll
    for (int i = 0; i < kI; ++i) {
      const float x[4] = {st[i][0], st[i][1], st[i][2], st[i][3]};
      const u32x4 w = split4(x);
      *reinterpret_cast<u32x2*>(hi_tile + n16 * 24 + 4 * jj) = u32x2{w[0], w[1]};
      *reinterpret_cast<u32x2*>(lo_tile + n16 * 24 + 4 * jj) = u32x2{w[2], w[3]};
      wave_sync();
      const u32x2 kh = __builtin_bit_cast(u32x2, tile_block_columns(hi_tile, 24, 4 * jj, 0, lane)), kl = __builtin_bit_cast(u32x2, tile_block_columns(lo_tile, 24, 4 * jj, 0, lane));
      wave_sync();
      unsigned char* const at = dst + (i * kS + s) * kPieceBytes + lane * 16 + 8 * half;
      *reinterpret_cast<u32x2*>(at) = kh;
      *reinterpret_cast<u32x2*>(at + kI * kS * kPieceBytes) = kl;
    }
    return;
  }
  if (STATES) __syncthreads();      // beside the one above
  if (!v_ok || (!STATES && p.seg_state)) return;
#pragma unroll
  for (int i = 0; i < kI; ++i)
    if (16 * i + 4 * jj < p.pitch) *reinterpret_cast<f32x4*>(state + 16 * i + 4 * jj) = st[i];
}

// A workgroup per (sequence, head, 16 value columns): S <- M S + C over the segments of the sequence.  Its waves share the rows of S; all of
// S goes round through LDS as operands.
constexpr int join_waves(int dp) { return dp / 16 < 4 ? dp / 16 : 4; }

template <int DP>
__global__ __launch_bounds__(64 * join_waves(DP)) void delta_join_kernel(const DeltaChunkArgs p) {
  using Sh = DeltaShape<DP>;
  constexpr int kS = Sh::kSteps, kI = Sh::kTiles, kMine = kI / join_waves(DP);
  __shared__ __align__(16) unsigned char ops[2][2][kS][kPieceBytes];      // two of them by turns: S hi, S lo
  const mops_hip_delta& a = p.a;
  const int heads = (int)a.heads, vd = (int)a.vd, blocks = (vd + 15) / 16;
  const int h = blockIdx.x / blocks % heads, b = blockIdx.x / blocks / heads;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, n16 = lane & 15, jj = lane >> 4, v0 = blockIdx.x % blocks * 16;
  const int slot = a.state_slots[b];
  if (slot < 0 || slot >= a.num_slots) return;
  const bool v_ok = v0 + n16 < vd, load_state = a.starts[b] > 0;
  const int v = v_ok ? v0 + n16 : vd - 1;
  float* const state = a.state + (((int64_t)slot * heads + h) * vd + v) * p.pitch;
  auto row = [&](int i) { return 16 * (wave * kMine + i) + 4 * jj; };      // of element 0 of this wave's tile i
  auto read = [&](const float* from, int i, bool on) {
    const bool ok = on && row(i) < p.pitch;
    const f32x4 w = *reinterpret_cast<const f32x4*>(from + (ok ? row(i) : 0));
    return ok ? w : f32x4{0.f, 0.f, 0.f, 0.f};
  };
  f32x4 st[kMine], next[kMine];
  u32x4 mh[kMine][kS], ml[kMine][kS];
  auto part = [&](int seg) { return p.seg_state + (((int64_t)seg * heads + h) * vd + v) * p.pitch; };
  auto fetch = [&](int seg) {
    const unsigned char* const map = p.seg_map + ((int64_t)seg * heads + h) * Sh::kMapBytes + lane * 16;
#pragma unroll
    for (int i = 0; i < kMine; ++i) {
      next[i] = read(part(seg), i, true);
#pragma unroll
      for (int s = 0; s < kS; ++s) {
        const int at = (wave * kMine + i) * kS + s;
        mh[i][s] = load16(map + at * kPieceBytes);
        ml[i][s] = load16(map + (kI * kS + at) * kPieceBytes);
      }
    }
  };
#pragma unroll
  for (int i = 0; i < kMine; ++i) st[i] = read(state, i, load_state);
  const int first = p.seq_segments[b], end = p.seq_segments[b + 1];
  if (first < end) fetch(first);
  for (int seg = first; seg < end; ++seg) {
    unsigned char(*const now)[kS][kPieceBytes] = ops[(seg - first) & 1];
#pragma unroll
    for (int i = 0; i < kMine; ++i) {
      const float x[4] = {st[i][0], st[i][1], st[i][2], st[i][3]};
      const u32x4 w = split4(x);
      const int tile = wave * kMine + i, at = lane * 16 + 8 * (tile & 1);
      *reinterpret_cast<u32x2*>(&now[0][tile >> 1][at]) = u32x2{w[0], w[1]};
      *reinterpret_cast<u32x2*>(&now[1][tile >> 1][at]) = u32x2{w[2], w[3]};
      if (v_ok && row(i) < p.pitch) *reinterpret_cast<f32x4*>(part(seg) + row(i)) = st[i];      // its lane has read C from there
    }
    __syncthreads();
#pragma unroll
    for (int s = 0; s < kS; ++s) {
      const bf16x8 hi = as_operand(load16(&now[0][s][lane * 16])), lo = as_operand(load16(&now[1][s][lane * 16]));
      const bool low = 32 * s < (int)a.d, high = 32 * s + 16 < (int)a.d;      // halves of the step that were written
#pragma unroll
      for (int i = 0; i < kMine; ++i) {
        u32x4 x = mh[i][s], y = ml[i][s];
        if (!low) x[0] = x[1] = y[0] = y[1] = 0u;
        if (!high) x[2] = x[3] = y[2] = y[3] = 0u;
        next[i] = mfma16(as_operand(x), hi, next[i]);
        next[i] = mfma16(as_operand(x), lo, next[i]);
        next[i] = mfma16(as_operand(y), hi, next[i]);
      }
    }
#pragma unroll
    for (int i = 0; i < kMine; ++i) st[i] = next[i];
    if (seg + 1 < end) fetch(seg + 1);
  }
  if (!v_ok) return;
#pragma unroll
  for (int i = 0; i < kMine; ++i)
    if (row(i) < p.pitch) *reinterpret_cast<f32x4*>(state + row(i)) = st[i];
}

int check_delta(const mops_hip_delta* a);      // delta_rule.hip

static int64_t operand_bytes(int64_t d) {
  if (d <= 32) return DeltaShape<32>::kBytes;
  if (d <= 64) return DeltaShape<64>::kBytes;
  return d <= 128 ? DeltaShape<128>::kBytes : DeltaShape<256>::kBytes;
}

static int64_t map_bytes(int64_t d) {
  if (d <= 32) return DeltaShape<32>::kMapBytes;
  if (d <= 64) return DeltaShape<64>::kMapBytes;
  return d <= 128 ? DeltaShape<128>::kMapBytes : DeltaShape<256>::kMapBytes;
}

template <int DP, int WAVES, bool STATES>
static int launch_scan(const DeltaChunkArgs& p, hipStream_t s) {
  constexpr int kLds = (int)(2 * (DeltaShape<DP>::kBytes - DeltaShape<DP>::from(STATES)));
  static const hipError_t lds = hipFuncSetAttribute(reinterpret_cast<const void*>(&delta_scan_kernel<DP, WAVES, STATES>), hipFuncAttributeMaxDynamicSharedMemorySize, kLds);
  if (lds != hipSuccess) return record_hip_error(lds);
  const int64_t columns = (p.a.vd + 15) / 16 * 16 + (STATES ? (p.a.d + 15) / 16 * 16 : 0);
  const int64_t total = p.num_segments * p.a.heads * ((columns + 16 * WAVES - 1) / (16 * WAVES));
  hipLaunchKernelGGL((delta_scan_kernel<DP, WAVES, STATES>), dim3((unsigned)((total + 7) / 8 * 8)), dim3(64 * WAVES), kLds, s, p);
  return finish_launch();
}

template <int DP>
static int launch_delta_chunks(const DeltaChunkArgs& p, hipStream_t s) {
  constexpr int kWaves = DP <= 128 ? 4 : 2, kMany = DP <= 128 ? 8 : 4;
  const int64_t items = (int64_t)p.num_chunks * p.a.heads;
  hipLaunchKernelGGL((delta_prepare_kernel<DP, kWaves>), dim3((unsigned)((items + kWaves - 1) / kWaves)), dim3(64 * kWaves), 0, s, p);
  // eight waves share a head's operands, four where eight leave most of the chip idle or the registers do not allow them
  const int64_t tiles = (p.a.vd + 15) / 16, rows = p.num_segments * p.a.heads;
  if (p.seg_state) {
    const int st = launch_scan<DP, kMany, true>(p, s);
    if (st != MOPS_HIP_OK) return st;
    hipLaunchKernelGGL((delta_join_kernel<DP>), dim3((unsigned)(p.a.batch * p.a.heads * tiles)), dim3(64 * join_waves(DP)), 0, s, p);
  }
  return tiles > 4 && rows * ((tiles + 7) / 8) >= 192 ? launch_scan<DP, kMany, false>(p, s) : launch_scan<DP, 4, false>(p, s);
}

}  // namespace mops

extern "C" int64_t mops_hip_delta_chunks_workspace_bytes(int64_t num_chunks, int64_t num_segments, int64_t batch, int64_t heads, int64_t d, int64_t vd) {
  using namespace mops;
  if (num_chunks <= 0 || heads <= 0 || d <= 0 || d > 256 || vd <= 0) return 0;
  const int64_t cut = num_segments > batch ? num_segments * heads * (map_bytes(d) + (vd * mops_hip_recurrence_state_pitch(d) * 4 + 15) / 16 * 16) : 0;
  return num_chunks * heads * operand_bytes(d) + cut;
}

extern "C" int64_t mops_hip_delta_chunks_workgroups(int64_t heads, int64_t vd) {
  return heads <= 0 || vd <= 0 ? MOPS_HIP_EINVAL : heads * ((vd + 127) / 128);
}

extern "C" int mops_hip_delta_chunks(const mops_hip_delta* a, const int32_t* chunks, int64_t num_chunks, const int32_t* segments, int64_t num_segments,
                                     const int32_t* seq_segments, void* workspace, int64_t workspace_bytes, void* stream) {
  using namespace mops;
  const int pre = check_delta(a);
  if (pre != 1) return pre;
  if (a->dtype != MOPS_HIP_BF16 || a->d > 256 || a->conv_weight) return MOPS_HIP_EUNSUPPORTED;
  if (num_chunks < 0 || num_segments < 0 || !chunks || !segments || !seq_segments || !a->cu_seqlens) return MOPS_HIP_EINVAL;
  if (num_chunks == 0 || num_segments == 0) return MOPS_HIP_OK;
  if (num_chunks * a->heads > 0x7fffffffLL || num_segments * a->heads * ((a->vd + a->d + 31) / 16) > 0x3fffffffLL ||
      a->batch * a->heads * ((a->vd + 15) / 16) > 0x7fffffffLL)
    return MOPS_HIP_EUNSUPPORTED;
  if (!workspace || workspace_bytes < mops_hip_delta_chunks_workspace_bytes(num_chunks, num_segments, a->batch, a->heads, a->d, a->vd)) return MOPS_HIP_EWORKSPACE;
  if (!aligned16(workspace)) return MOPS_HIP_EALIGN;
  DeltaChunkArgs p;
  p.a = *a;
  p.chunks = chunks;
  p.segments = segments;
  p.seq_segments = seq_segments;
  p.num_chunks = (int)num_chunks;
  p.num_segments = (int)num_segments;
  p.pitch = (int)mops_hip_recurrence_state_pitch(a->d);
  p.operands = (unsigned char*)workspace;
  p.seg_map = p.operands + num_chunks * a->heads * operand_bytes(a->d);
  p.seg_state = num_segments > a->batch ? (float*)(p.seg_map + num_segments * a->heads * map_bytes(a->d)) : nullptr;
  p.vec = a->d % 4 == 0 && a->vd % 4 == 0 && a->q_stride % 4 == 0 && a->k_stride % 4 == 0 && a->log_decay_stride % 4 == 0 && a->out_stride % 4 == 0 &&
          aligned16(a->q) && aligned16(a->k) && aligned16(a->log_decay) && aligned16(a->out);
  hipStream_t s = (hipStream_t)stream;
  if (a->d <= 32) return launch_delta_chunks<32>(p, s);
  if (a->d <= 64) return launch_delta_chunks<64>(p, s);
  return a->d <= 128 ? launch_delta_chunks<128>(p, s) : launch_delta_chunks<256>(p, s);
}
