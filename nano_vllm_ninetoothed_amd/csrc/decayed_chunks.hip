// The recurrence of decayed_recurrence.hip for portions of many tokens, 64 tokens at a time on the matrix cores (bf16 in,
// float32 accumulation and state):
//
//   L_i = sum of log a over the chunk up to token i,  s = input scale
//   O_i = e^{L_i} S^T q_i + sum_{j <= i} e^{L_i - L_j} s_j (q_i . k_j) v_j + skip v_i
//   S  <- e^{L_end} S + sum_j e^{L_end - L_j} s_j k_j v_j^T
//
// Workgroup = (segment, head, tile of VT value columns), walking the chunks of its segment with S [d x VT] in the
// accumulators.  All products are v_mfma_f32_32x32x16_bf16:
//   P^T [j, i] = K Q^T                 rows of the two LDS tiles as they are
//   O^T [v, i] = S^T Q^T + V^T P^T     the accumulator layout of P^T is the B-operand layout of the second product, up to
//                                      the order of the tokens inside a step, which V^T takes over
//   S [d, v] += K^T (w V)              both operands through transposing LDS reads (ds_read_b64_tr_b16)
// What the recurrence keeps in 32 bits - the state, the decayed scores, the decayed values - enters a product as the sum of two
// bf16 numbers (value = hi + lo, 16 significant bits), at the price of a second MFMA.
//
// A sequence is one segment when there are enough sequences and heads to fill the chip.  Otherwise it is cut:
//   pass 1 (STATE_ONLY)  every segment from a zero state: its contribution and its total decay
//   pass 2 (scan)        the state at the start of every segment, and the final state into the sequence's slot
//   pass 3               every segment again, with outputs, from its start state
#include "mfma_tiles.h"

namespace mops {

constexpr int kChunk = 64;

struct ChunkArgs {
  const uint16_t *q, *k, *v, *dt;
  int64_t q_stride, k_stride, v_stride, dt_stride;
  uint16_t* out;
  int64_t out_stride;
  float* state;
  int64_t num_slots;
  const int32_t *state_slots, *cu_seqlens, *starts;
  const int32_t* segments;      // [n][3]: sequence, first token, one past the last
  int num_segments;
  int heads, groups, d, vd, pitch;
  const float *log_decay, *dt_bias, *neg_a, *skip, *cos_sin;
  int rot;
  int64_t max_positions;
  float k_scale;
  float* seg_state;             // [n][heads][vd][pitch], or nullptr: one segment per sequence
  float* seg_decay;             // [n][heads]: natural logarithm of the segment's total decay
};

template <int DP, int VT>
struct ChunkShape {
  static constexpr int kThreads = VT * 4;                 // a wave per 32 x 32 tile of [VT, 64 tokens]
  static constexpr int kPitch = DP + 8;                   // elements; keeps 16-byte rows off each other's banks
  static constexpr int kVPitch = VT + 8;
  static constexpr int kQ = kChunk * kPitch, kV = kChunk * kVPitch, kS = VT * kPitch;
  static constexpr int bytes(bool state_only) { return ((state_only ? 0 : kQ + 2 * kS) + kQ + kV) * 2 + (3 * kChunk + 32) * 4; }
};

// q, k and v rows of a chunk on their way from memory into the LDS tiles: q and k rotated, scaled and rounded to bf16, zeros
// outside the chunk and the head.  fetch() issues every load of a chunk at once, so that it can be called while the chunk
// before is still being worked on; store() finishes the values and writes the tiles.
// A thread owns pairs of 16-byte pieces of a row, for q and k alike: pair p < rot / 16 is columns (8p, 8p + rot/2), which
// rotate with each other; the pairs behind take two pieces that pass unchanged.
template <int DP, int VT, bool STATE_ONLY, int PAIRS>
struct ChunkLoader {
  static constexpr int kThreads = ChunkShape<DP, VT>::kThreads, kPitch = DP + 8, kVPitch = VT + 8;
  static constexpr int kVPieces = kChunk * (VT / 8) / kThreads;
  u32x4 k[PAIRS][2], q[STATE_ONLY ? 1 : PAIRS][2], v[kVPieces];
  float cs[PAIRS][8], sn[PAIRS][8];

  static __device__ __forceinline__ bool place(int i, const ChunkArgs& a, int& r, int& c0, int& c1, bool& rotates) {
    r = i / (DP / 16);
    const int p = i % (DP / 16), half = a.rot >> 1;
    rotates = 8 * p < half;
    c0 = rotates ? 8 * p : 16 * p;       // behind the rotated pairs: rot + 16 (p - rot / 16) = 16 p
    c1 = rotates ? c0 + half : c0 + 8;
    return i < kChunk * (DP / 16);
  }
  __device__ __forceinline__ void fetch_qk(int first, const uint16_t* kp, const uint16_t* qp, int n, const ChunkArgs& a) {
#pragma unroll
    for (int j = 0; j < PAIRS; ++j) {
      int r, c0, c1;
      bool rotates;
      const bool in = place((first + j) * kThreads + (int)threadIdx.x, a, r, c0, c1, rotates) && r < n;
      const u32x4 zero = {0u, 0u, 0u, 0u};
      k[j][0] = in && c0 < a.d ? load16(kp + r * a.k_stride + c0) : zero;
      k[j][1] = in && c1 < a.d ? load16(kp + r * a.k_stride + c1) : zero;
      if (!STATE_ONLY) {
        q[j][0] = in && c0 < a.d ? load16(qp + r * a.q_stride + c0) : zero;
        q[j][1] = in && c1 < a.d ? load16(qp + r * a.q_stride + c1) : zero;
      }
    }
  }
  __device__ __forceinline__ void fetch_trig(int first, int n, int pos0, const ChunkArgs& a) {
#pragma unroll
    for (int j = 0; j < PAIRS; ++j) {
      int r, c0, c1;
      bool rotates;
      const bool in = place((first + j) * kThreads + (int)threadIdx.x, a, r, c0, c1, rotates) && r < n;
      if (in && rotates) {
        const int64_t pos = pos0 + r < a.max_positions ? pos0 + r : a.max_positions - 1;
        load_vec<8>(a.cos_sin + pos * a.rot + c0, cs[j]);
        load_vec<8>(a.cos_sin + pos * a.rot + (a.rot >> 1) + c0, sn[j]);
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          cs[j][e] = 1.f;
          sn[j][e] = 0.f;
        }
      }
    }
  }
  __device__ __forceinline__ void fetch_v(const uint16_t* vp, int n, int vlen, const ChunkArgs& a) {
#pragma unroll
    for (int j = 0; j < kVPieces; ++j) {
      const int i = j * kThreads + (int)threadIdx.x, r = i / (VT / 8), c = (i % (VT / 8)) * 8;
      v[j] = r < n && c < vlen ? load16(vp + r * a.v_stride + c) : u32x4{0u, 0u, 0u, 0u};
    }
  }
  static __device__ __forceinline__ void finish(uint16_t* tile, int at0, int at1, const u32x4 (&w)[2], const float (&cs)[8], const float (&sn)[8],
                                                float scale) {
    u32x4 o0, o1;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float x0 = bf16lo_to_f32(w[0][e]), x1 = bf16hi_to_f32(w[0][e]), y0 = bf16lo_to_f32(w[1][e]), y1 = bf16hi_to_f32(w[1][e]);
      o0[e] = pack_bf16x2((x0 * cs[2 * e] - y0 * sn[2 * e]) * scale, (x1 * cs[2 * e + 1] - y1 * sn[2 * e + 1]) * scale);
      o1[e] = pack_bf16x2((y0 * cs[2 * e] + x0 * sn[2 * e]) * scale, (y1 * cs[2 * e + 1] + x1 * sn[2 * e + 1]) * scale);
    }
    store16(tile + at0, o0);
    store16(tile + at1, o1);
  }
  __device__ __forceinline__ void store_qk(int first, uint16_t* tk, uint16_t* tq, const ChunkArgs& a) const {
#pragma unroll
    for (int j = 0; j < PAIRS; ++j) {
      int r, c0, c1;
      bool rotates;
      if (!place((first + j) * kThreads + (int)threadIdx.x, a, r, c0, c1, rotates)) continue;
      finish(tk, r * kPitch + c0, r * kPitch + c1, k[j], cs[j], sn[j], a.k_scale);
      if (!STATE_ONLY) finish(tq, r * kPitch + c0, r * kPitch + c1, q[j], cs[j], sn[j], 1.f);
    }
  }
  __device__ __forceinline__ void store_v(uint16_t* tv) const {
#pragma unroll
    for (int j = 0; j < kVPieces; ++j) {
      const int i = j * kThreads + (int)threadIdx.x;
      store16(tv + i / (VT / 8) * kVPitch + (i % (VT / 8)) * 8, v[j]);
    }
  }
};

// The same for any alignment, element by element.
template <int DP, int THREADS>
__device__ __forceinline__ void load_tile_scalar(uint16_t* tile, const uint16_t* src, int64_t stride, int n, int pos0, const ChunkArgs& a, float scale) {
  const int half = a.rot >> 1;
#pragma unroll 1
  for (int i = threadIdx.x; i < kChunk * DP; i += THREADS) {
    const int r = i / DP, c = i % DP;
    float x = 0.f;
    if (r < n && c < a.d) {
      x = bf16lo_to_f32(src[r * stride + c]);
      if (c < a.rot) {
        const bool lower = c < half;
        const float mate = bf16lo_to_f32(src[r * stride + (lower ? c + half : c - half)]);
        const int64_t pos = pos0 + r < a.max_positions ? pos0 + r : a.max_positions - 1;
        const float* trig = a.cos_sin + pos * a.rot + (lower ? c : c - half);
        x = x * trig[0] + (lower ? -mate : mate) * trig[half];
      }
      x *= scale;
    }
    tile[r * (DP + 8) + c] = (uint16_t)f32_to_bf16_bits(x);
  }
}

template <int DP, int VT, bool STATE_ONLY, bool VEC>
__global__ __launch_bounds__(VT * 4, 2) void decayed_chunk_kernel(const ChunkArgs a) {
  using S = ChunkShape<DP, VT>;
  constexpr int kVTiles = VT / 32;
  constexpr int kDTiles = DP >= 64 ? DP / 64 : 1;         // 32-wide tiles of d per wave in the state
  extern __shared__ __align__(16) unsigned char smem[];
  uint16_t* const tk = reinterpret_cast<uint16_t*>(smem);
  uint16_t* const tv = tk + S::kQ;
  uint16_t* const tq = tv + S::kV;
  uint16_t* const ts_hi = tq + S::kQ;
  uint16_t* const ts_lo = ts_hi + S::kS;
  float* const cum = reinterpret_cast<float*>(STATE_ONLY ? tq : ts_lo + S::kS);   // [64] L, base 2
  float* const scl = cum + kChunk;                                                  // [64] input scale
  float* const wgt0 = scl + 2 * kChunk;                                             // [32] scale * 2^(L_31 - L)
  float* const wgt = scl + kChunk;                                                  // [64] scale * 2^(L_end - L)

  // consecutive workgroups go to different XCDs: give each XCD a contiguous run of items, so that the tiles and heads that
  // read the same q and k rows share an L2
  const int vtiles = (a.vd + VT - 1) / VT;
  const int total = a.num_segments * a.heads * vtiles;
  const int per_xcd = (total + 7) / 8;
  const int item = (blockIdx.x % 8) * per_xcd + blockIdx.x / 8;
  if (blockIdx.x / 8 >= per_xcd || item >= total) return;
  const int v0 = (item % vtiles) * VT;
  const int h = (item / vtiles) % a.heads;
  const int seg = item / (vtiles * a.heads);
  const int b = a.segments[3 * seg], t_begin = a.segments[3 * seg + 1], t_end = a.segments[3 * seg + 2];
  const int slot = a.state_slots[b], start = a.starts[b], seq_begin = a.cu_seqlens[b];
  if (slot < 0 || slot >= a.num_slots) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x / 64;
  const int col = lane & 31, hh = lane >> 5;
  const int vt = wave % kVTiles, half_id = wave / kVTiles;   // half_id: which 32 tokens, and which half of d
  const int g = h / (a.heads / a.groups);
  const uint16_t *qp = a.q + (int64_t)g * a.d, *kp = a.k + (int64_t)g * a.d, *vp = a.v + (int64_t)h * a.vd + v0;
  const int vlen = a.vd - v0 < VT ? a.vd - v0 : VT;
  const float skip = a.skip ? a.skip[h] : 0.f;
  constexpr float kLog2e = 1.4426950408889634f;
  const float la_const = a.log_decay ? a.log_decay[h] * kLog2e : 0.f;
  const float dt_bias = a.dt ? a.dt_bias[h] : 0.f, neg_a = a.dt ? a.neg_a[h] * kLog2e : 0.f;

  // S: rows d = 32 (half_id kDTiles + i) + 8 q + 4 hh + e (four consecutive ones per q), column v0 + 32 vt + (lane & 31)
  f32x16 st[kDTiles];
  const bool has_state_tile = half_id * kDTiles * 32 < DP;
  const int v_col = 32 * vt + col;
  auto state_d = [&](int i, int q4) { return 32 * (half_id * kDTiles + i) + 8 * q4 + 4 * hh; };
  float* gstate = nullptr;
  bool load_state = false;
  if (!STATE_ONLY) {
    if (a.seg_state) {
      gstate = a.seg_state + (((int64_t)seg * a.heads + h) * a.vd + v0) * a.pitch;
      load_state = true;
    } else {
      gstate = a.state + (((int64_t)slot * a.heads + h) * a.vd + v0) * a.pitch;
      load_state = start > 0;
    }
  }
#pragma unroll
  for (int i = 0; i < kDTiles; ++i)
#pragma unroll
    for (int q4 = 0; q4 < 4; ++q4) {
      // no branch per element (the accumulators would be copied at each): every lane reads some valid element, then selects
      const bool ok = load_state && state_d(i, q4) < a.pitch && v_col < vlen;
      f32x4 x = {0.f, 0.f, 0.f, 0.f};
      if (!STATE_ONLY) x = *reinterpret_cast<const f32x4*>(gstate + (ok ? v_col * a.pitch + state_d(i, q4) : 0));
#pragma unroll
      for (int e = 0; e < 4; ++e) st[i][4 * q4 + e] = ok ? x[e] : 0.f;
    }

  constexpr int kPairsAll = (kChunk * (DP / 16) + S::kThreads - 1) / S::kThreads;
  constexpr bool kAhead = VEC && kPairsAll <= 2;          // a whole chunk fits the registers next to the accumulators
  constexpr int kPairs = kPairsAll <= 2 ? kPairsAll : 2;
  ChunkLoader<DP, VT, STATE_ONLY, kPairs> ld;
  float dt_next = 0.f;
  auto fetch = [&](int t) {
    const int m = t_end - t < kChunk ? t_end - t : kChunk;
    ld.fetch_qk(0, kp + (int64_t)t * a.k_stride, qp + (int64_t)t * a.q_stride, m, a);
    ld.fetch_trig(0, m, start + (t - seq_begin), a);
    ld.fetch_v(vp + (int64_t)t * a.v_stride, m, vlen, a);
  };
  auto fetch_dt = [&](int t) { dt_next = a.dt && wave == 0 && t + lane < t_end ? bf16lo_to_f32(a.dt[(int64_t)(t + lane) * a.dt_stride + h]) : 0.f; };
  if (kAhead) fetch(t_begin);
  fetch_dt(t_begin);
  float total_log = 0.f;
  for (int t0 = t_begin; t0 < t_end; t0 += kChunk) {
    const int n = t_end - t0 < kChunk ? t_end - t0 : kChunk;
    const int pos0 = start + (t0 - seq_begin);
    __syncthreads();     // the last chunk's tiles have been read
    if (kAhead) {
      ld.store_qk(0, tk, tq, a);
      ld.store_v(tv);
    } else if (VEC) {
      ld.fetch_v(vp + (int64_t)t0 * a.v_stride, n, vlen, a);
#pragma unroll 1
      for (int first = 0; first < kPairsAll; first += kPairs) {
        ld.fetch_qk(first, kp + (int64_t)t0 * a.k_stride, qp + (int64_t)t0 * a.q_stride, n, a);
        ld.fetch_trig(first, n, pos0, a);
        ld.store_qk(first, tk, tq, a);
      }
      ld.store_v(tv);
    } else {
      load_tile_scalar<DP, S::kThreads>(tk, kp + (int64_t)t0 * a.k_stride, a.k_stride, n, pos0, a, a.k_scale);
      if (!STATE_ONLY) load_tile_scalar<DP, S::kThreads>(tq, qp + (int64_t)t0 * a.q_stride, a.q_stride, n, pos0, a, 1.f);
#pragma unroll 1
      for (int i = threadIdx.x; i < kChunk * VT; i += S::kThreads) {
        const int r = i / VT, c = i % VT;
        tv[r * S::kVPitch + c] = r < n && c < vlen ? vp[(int64_t)(t0 + r) * a.v_stride + c] : (uint16_t)0;
      }
    }
    if (wave == 0) {     // decays of the chunk: lane = token
      float la = 0.f, s = 0.f, l;
      if (a.dt) {
        if (lane < n) {
          s = softplus_f32(dt_next + dt_bias);
          la = neg_a * s;
        }
        l = la;
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
          const float up = __shfl_up(l, off, 64);
          if (lane >= off) l += up;
        }
      } else {
        s = lane < n ? 1.f : 0.f;
        l = la_const * (float)(lane + 1 < n ? lane + 1 : n);
      }
      const float l_end = __shfl(l, 63, 64);
      cum[lane] = l;
      scl[lane] = s;
      wgt[lane] = s * __builtin_amdgcn_exp2f(l_end - l);
      const float l_mid = __shfl(l, 31, 64);
      if (lane < 32) wgt0[lane] = s * __builtin_amdgcn_exp2f(l_mid - l);
    }
    if (!STATE_ONLY && has_state_tile) {
#pragma unroll
      for (int i = 0; i < kDTiles; ++i)
#pragma unroll
        for (int q4 = 0; q4 < 4; ++q4) {
          const uint32_t h0 = pack_bf16x2(st[i][4 * q4], st[i][4 * q4 + 1]), h1 = pack_bf16x2(st[i][4 * q4 + 2], st[i][4 * q4 + 3]);
          const uint32_t l0 = pack_bf16x2(st[i][4 * q4] - bf16lo_to_f32(h0), st[i][4 * q4 + 1] - bf16hi_to_f32(h0));
          const uint32_t l1 = pack_bf16x2(st[i][4 * q4 + 2] - bf16lo_to_f32(h1), st[i][4 * q4 + 3] - bf16hi_to_f32(h1));
          *reinterpret_cast<u32x2*>(ts_hi + v_col * S::kPitch + state_d(i, q4)) = u32x2{h0, h1};
          *reinterpret_cast<u32x2*>(ts_lo + v_col * S::kPitch + state_d(i, q4)) = u32x2{l0, l1};
        }
    }
    __syncthreads();
    const float l_end = cum[kChunk - 1];
    total_log += l_end;
    const bool more = t0 + kChunk < t_end;
    if (more) fetch_dt(t0 + kChunk);

    if (!STATE_ONLY) {
      const int i_tok = 32 * half_id + col;      // this lane's output token
      const float l_i = cum[i_tok];
      f32x16 o;
#pragma unroll
      for (int r = 0; r < 16; ++r) o[r] = 0.f;
#pragma unroll
      for (int kk = 0; kk < DP / 16; ++kk) {
        const bf16x8 qb = tile_row(tq, S::kPitch, i_tok, 16 * kk + 8 * hh);
        o = mfma32(tile_row(ts_hi, S::kPitch, 32 * vt + col, 16 * kk + 8 * hh), qb, o);
        o = mfma32(tile_row(ts_lo, S::kPitch, 32 * vt + col, 16 * kk + 8 * hh), qb, o);
      }
      const float e_i = __builtin_amdgcn_exp2f(l_i), e_mid = __builtin_amdgcn_exp2f(half_id ? l_i - cum[31] : 0.f);
#pragma unroll
      for (int r = 0; r < 16; ++r) o[r] *= e_i;
      for (int jt = 0; jt <= half_id; ++jt) {
        f32x16 p;
#pragma unroll
        for (int r = 0; r < 16; ++r) p[r] = 0.f;
#pragma unroll
        for (int kk = 0; kk < DP / 16; ++kk)
          p = mfma32(tile_row(tk, S::kPitch, 32 * jt + col, 16 * kk + 8 * hh), tile_row(tq, S::kPitch, i_tok, 16 * kk + 8 * hh), p);
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
          const int j0 = 32 * jt + 16 * ks + 4 * hh;       // tokens j0 .. j0+3 and j0+8 .. j0+11
          float pv[8];
#pragma unroll
          for (int e = 0; e < 8; ++e) {
            const int j = j0 + (e & 3) + 8 * (e >> 2);
            // below the diagonal tile the weight is a product of one factor per token on either side of the tile border
            if (jt < half_id) pv[e] = p[8 * ks + e] * (wgt0[j] * e_mid);
            else pv[e] = j <= i_tok ? p[8 * ks + e] * (scl[j] * __builtin_amdgcn_exp2f(l_i - cum[j])) : 0.f;
          }
          bf16x8 hi, lo;
          split8(pv, hi, lo);
          const bf16x8 va = __builtin_bit_cast(bf16x8, tile_columns(tv, S::kVPitch, j0, j0 + 8, 32 * vt, lane));
          o = mfma32(va, hi, o);
          o = mfma32(va, lo, o);
        }
      }
      if (skip != 0.f) {
#pragma unroll
        for (int q4 = 0; q4 < 4; ++q4)
#pragma unroll
          for (int e = 0; e < 4; ++e)
            o[4 * q4 + e] += skip * bf16lo_to_f32(tv[i_tok * S::kVPitch + 32 * vt + 8 * q4 + 4 * hh + e]);
      }
      uint16_t* orow = a.out + (int64_t)(t0 + i_tok) * a.out_stride + (int64_t)h * a.vd + v0;
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        // eight consecutive columns per lane: the lower half of the wave completes piece 2 half, the upper half 2 half + 1
        const u32x2 even = {pack_bf16x2(o[8 * half], o[8 * half + 1]), pack_bf16x2(o[8 * half + 2], o[8 * half + 3])};
        const u32x2 odd = {pack_bf16x2(o[8 * half + 4], o[8 * half + 5]), pack_bf16x2(o[8 * half + 6], o[8 * half + 7])};
        const u32x2 mine = hh ? odd : even, give = hh ? even : odd;
        const u32x2 got = {(uint32_t)__shfl_xor((int)give[0], 32, 64), (uint32_t)__shfl_xor((int)give[1], 32, 64)};
        const u32x4 w = hh ? u32x4{got[0], got[1], mine[0], mine[1]} : u32x4{mine[0], mine[1], got[0], got[1]};
        const int v = 32 * vt + 16 * half + 8 * hh;
        if (i_tok < n) {
          if (VEC) {
            if (v < vlen) store16(orow + v, w);
          } else {
#pragma unroll
            for (int e = 0; e < 8; ++e)
              if (v + e < vlen) orow[v + e] = (uint16_t)(w[e >> 1] >> (16 * (e & 1)));
          }
        }
      }
    }
    // the next chunk is on its way while the state takes this one in
    if (kAhead && more) fetch(t0 + kChunk);
    // ---- S <- e^{L_end} S + K^T (w V)
    if (has_state_tile) {
      const float e_end = __builtin_amdgcn_exp2f(l_end);
#pragma unroll
      for (int i = 0; i < kDTiles; ++i)
#pragma unroll
        for (int r = 0; r < 16; ++r) st[i][r] *= e_end;
#pragma unroll
      for (int ks = 0; ks < kChunk / 16; ++ks) {
        const int j0 = 16 * ks + 4 * hh;
        const s16x8 raw = tile_columns(tv, S::kVPitch, j0, j0 + 8, 32 * vt, lane);
        float x[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = bf16lo_to_f32((uint16_t)raw[e]) * wgt[j0 + (e & 3) + 8 * (e >> 2)];
        bf16x8 hi, lo;
        split8(x, hi, lo);
#pragma unroll
        for (int i = 0; i < kDTiles; ++i) {
          const bf16x8 ka = __builtin_bit_cast(bf16x8, tile_columns(tk, S::kPitch, j0, j0 + 8, 32 * (half_id * kDTiles + i), lane));
          st[i] = mfma32(ka, hi, st[i]);
          st[i] = mfma32(ka, lo, st[i]);
        }
      }
    }
  }

  float* dst = nullptr;
  if (STATE_ONLY) dst = a.seg_state + (((int64_t)seg * a.heads + h) * a.vd + v0) * a.pitch;
  else if (!a.seg_state) dst = gstate;
  if (dst && has_state_tile) {
#pragma unroll
    for (int i = 0; i < kDTiles; ++i)
#pragma unroll
      for (int q4 = 0; q4 < 4; ++q4)
        if (v_col < vlen && state_d(i, q4) < a.pitch)
          *reinterpret_cast<f32x4*>(dst + v_col * a.pitch + state_d(i, q4)) = f32x4{st[i][4 * q4], st[i][4 * q4 + 1], st[i][4 * q4 + 2], st[i][4 * q4 + 3]};
  }
  if (STATE_ONLY && v0 == 0 && threadIdx.x == 0) a.seg_decay[(int64_t)seg * a.heads + h] = total_log;
}

// Start state of every segment (in place of its contribution) and the final state of every sequence.  Segments of a sequence
// are consecutive; seq_segments[b], seq_segments[b + 1] bound them.
__global__ __launch_bounds__(256) void decayed_segment_scan_kernel(const ChunkArgs a, const int32_t* __restrict__ seq_segments) {
  const int h = blockIdx.y, b = blockIdx.z;
  const int64_t n = (int64_t)a.vd * a.pitch;
  const int64_t e = ((int64_t)blockIdx.x * 256 + threadIdx.x) * 4;
  const int slot = a.state_slots[b];
  if (e >= n || slot < 0 || slot >= a.num_slots) return;
  float* gs = a.state + ((int64_t)slot * a.heads + h) * n + e;
  f32x4 s = {0.f, 0.f, 0.f, 0.f};
  if (a.starts[b] > 0) s = *reinterpret_cast<const f32x4*>(gs);
  for (int seg = seq_segments[b]; seg < seq_segments[b + 1]; ++seg) {
    float* p = a.seg_state + ((int64_t)seg * a.heads + h) * n + e;
    const f32x4 u = *reinterpret_cast<const f32x4*>(p);
    const float decay = __builtin_amdgcn_exp2f(a.seg_decay[(int64_t)seg * a.heads + h]);
    *reinterpret_cast<f32x4*>(p) = s;
#pragma unroll
    for (int i = 0; i < 4; ++i) s[i] = decay * s[i] + u[i];
  }
  *reinterpret_cast<f32x4*>(gs) = s;
}

template <int DP, int VT, bool VEC>
static int launch_chunks(const ChunkArgs& a, const int32_t* seq_segments, int64_t batch, hipStream_t s) {
  using S = ChunkShape<DP, VT>;
  const int64_t items = (int64_t)a.num_segments * a.heads * ((a.vd + VT - 1) / VT);
  const dim3 grid((unsigned)((items + 7) / 8 * 8)), block(S::kThreads);
  static const hipError_t lds = hipFuncSetAttribute(reinterpret_cast<const void*>(&decayed_chunk_kernel<DP, VT, false, VEC>),
                                                    hipFuncAttributeMaxDynamicSharedMemorySize, S::bytes(false));
  static const hipError_t lds_state = hipFuncSetAttribute(reinterpret_cast<const void*>(&decayed_chunk_kernel<DP, VT, true, VEC>),
                                                          hipFuncAttributeMaxDynamicSharedMemorySize, S::bytes(true));
  if (lds != hipSuccess) return record_hip_error(lds);
  if (lds_state != hipSuccess) return record_hip_error(lds_state);
  if (a.seg_state) {
    hipLaunchKernelGGL((decayed_chunk_kernel<DP, VT, true, VEC>), grid, block, S::bytes(true), s, a);
    const int64_t quads = ((int64_t)a.vd * a.pitch / 4 + 255) / 256;
    hipLaunchKernelGGL(decayed_segment_scan_kernel, dim3((unsigned)quads, (unsigned)a.heads, (unsigned)batch), dim3(256), 0, s, a, seq_segments);
  }
  hipLaunchKernelGGL((decayed_chunk_kernel<DP, VT, false, VEC>), grid, block, S::bytes(false), s, a);
  return finish_launch();
}

}  // namespace mops

extern "C" int mops_hip_decayed_chunks(const mops_hip_recurrence* r, const int32_t* segments, int64_t num_segments,
                                       const int32_t* seq_segments, float* seg_state, float* seg_decay, void* stream) {
  using namespace mops;
  if (!r || r->batch < 0 || num_segments < 0) return MOPS_HIP_EINVAL;
  if (r->batch == 0 || num_segments == 0) return MOPS_HIP_OK;
  if (r->dtype != MOPS_HIP_BF16 || r->conv_weight) return MOPS_HIP_EUNSUPPORTED;
  if (!r->q || !r->k || !r->v || !r->out || !r->state || !r->state_slots || !r->starts || !r->cu_seqlens || !segments) return MOPS_HIP_EINVAL;
  if (!seg_state != !seg_decay || (seg_state && !seq_segments) || (!seg_state && num_segments > r->batch)) return MOPS_HIP_EINVAL;
  if (r->heads <= 0 || r->groups <= 0 || r->heads % r->groups || r->d <= 0 || r->vd <= 0 || r->num_slots <= 0) return MOPS_HIP_EINVAL;
  if (r->d > 256 || r->heads > 65535 || r->batch > 65535 || r->vd > 65536) return MOPS_HIP_EUNSUPPORTED;
  if (r->q_stride < r->groups * r->d || r->k_stride < r->groups * r->d || r->v_stride < r->heads * r->vd || r->out_stride < r->heads * r->vd)
    return MOPS_HIP_EINVAL;
  if (!r->log_decay == !r->dt) return MOPS_HIP_EINVAL;
  if (r->dt && (!r->dt_bias || !r->neg_a || r->dt_stride < r->heads)) return MOPS_HIP_EINVAL;
  if (r->rot < 0 || (r->rot & 1) || r->rot > r->d || (r->rot && (!r->cos_sin || r->max_positions <= 0))) return MOPS_HIP_EINVAL;
  if (!aligned16(r->state) || (seg_state && !aligned16(seg_state))) return MOPS_HIP_EALIGN;
  if (num_segments * r->heads * ((r->vd + 31) / 32) > 0x3fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  ChunkArgs a;
  a.q = (const uint16_t*)r->q; a.k = (const uint16_t*)r->k; a.v = (const uint16_t*)r->v; a.dt = (const uint16_t*)r->dt;
  a.q_stride = r->q_stride; a.k_stride = r->k_stride; a.v_stride = r->v_stride; a.dt_stride = r->dt_stride;
  a.out = (uint16_t*)r->out; a.out_stride = r->out_stride;
  a.state = r->state; a.num_slots = r->num_slots;
  a.state_slots = r->state_slots; a.cu_seqlens = r->cu_seqlens; a.starts = r->starts;
  a.segments = segments; a.num_segments = (int)num_segments;
  a.heads = (int)r->heads; a.groups = (int)r->groups; a.d = (int)r->d; a.vd = (int)r->vd;
  a.pitch = (int)mops_hip_recurrence_state_pitch(r->d);
  a.log_decay = r->log_decay; a.dt_bias = r->dt_bias; a.neg_a = r->neg_a; a.skip = r->skip; a.cos_sin = r->cos_sin;
  a.rot = (int)r->rot; a.max_positions = r->max_positions; a.k_scale = r->k_scale;
  a.seg_state = seg_state; a.seg_decay = seg_decay;
  const bool vec = r->d % 8 == 0 && r->q_stride % 8 == 0 && r->k_stride % 8 == 0 && aligned16(r->q) && aligned16(r->k) &&
                   (r->rot == 0 || (r->rot % 16 == 0 && aligned16(r->cos_sin))) && r->vd % 8 == 0 && r->v_stride % 8 == 0 &&
                   r->out_stride % 8 == 0 && aligned16(r->v) && aligned16(r->out);
  hipStream_t s = (hipStream_t)stream;
  if (!vec) return a.d <= 64 ? launch_chunks<64, 64, false>(a, seq_segments, r->batch, s) : launch_chunks<256, 64, false>(a, seq_segments, r->batch, s);
#define MOPS_CHUNKS(D) (a.vd <= 32 ? launch_chunks<D, 32, true>(a, seq_segments, r->batch, s) : launch_chunks<D, 64, true>(a, seq_segments, r->batch, s))
  if (a.d <= 32) return MOPS_CHUNKS(32);
  if (a.d <= 64) return MOPS_CHUNKS(64);
  if (a.d <= 128) return MOPS_CHUNKS(128);
  return MOPS_CHUNKS(256);
#undef MOPS_CHUNKS
}
