// The recurrence with a decay per key channel (decayed_recurrence.hip) for portions of many tokens, 16 tokens at a time on the
// matrix cores (bf16 in, float32 accumulation and state).  With L_t = log2 of the product of the decays of a chunk up to token t
// (per channel; L_-1 = 0, L_15 = the whole chunk) and S the state in front of the chunk:
//
//   o_t = S^T (2^{L_{t-1}} r_t) + sum_{j<t} P[t, j] v_j + (r_t . u k_t) v_t,   P[t, j] = sum_d r_t[d] k_j[d] 2^{L_{t-1}[d] - L_j[d]}
//   S  <- 2^{L_15} S + sum_j (2^{L_15 - L_j} k_j) v_j^T
//
// P is a product of one factor per token on either side of a reference: 2^{L_{t-1} - ref} r_t and 2^{ref - L_j} k_j.  The reference
// is L_7 where t >= 8 > j, so that both exponents are negative, and the middle of the half chunk (L_3, L_11) where t and j lie in
// the same half: at most four decays lie between a token and its reference, so an exponent stays below 4 * 28.  (A decay below
// 2^-28 counts as 2^-28: what it leaves of a number is less than that number's last bit in float32.)
//
// Workgroup (four waves) = (segment, head, 64 NV value columns).  A chunk has two steps with one barrier (or two) between:
//   scaled rows   lane = token of a 16-lane row, which owns DP / 16 channels: L by a scan over the row, all factors, and the five
//                 scaled copies of r and k as the sum of two bf16 numbers (value = hi + lo, 16 significant bits) into LDS.
//                 The next chunk's loads are issued behind this step.
//   products      a wave owns 16 NV value columns with S [d x 16 NV] in its accumulators; v_mfma_f32_16x16x32_bf16:
//       P^T [j, t]              every wave, redundantly
//       O^T [v, t] = S^T r + V^T P^T   S straight from the accumulators: their layout is an operand layout up to the order of the
//                                      d's, which the reads of r follow; hi and lo of P^T share one product (16 + 16 deep)
//       S [d, v]  += k^T V             hi and lo of k likewise
//
// One segment per sequence, or segments in three passes as in decayed_chunks.hip: states from zero, scan, outputs.
#include "mfma_tiles.h"

namespace mops {

constexpr int kCTokens = 16;
constexpr float kLeastLog2Decay = -28.f;

struct ChannelArgs {
  const uint16_t *r, *k, *v;
  const float *log_decay, *bonus;
  int64_t r_stride, k_stride, v_stride, decay_stride;
  uint16_t* out;
  int64_t out_stride;
  float* state;
  int64_t num_slots;
  const int32_t *state_slots, *cu_seqlens, *starts;
  const int32_t* segments;      // [n][3]: sequence, first token, one past the last
  int num_segments;
  int heads, d, vd, pitch;
  float* seg_state;             // [n][heads][vd][pitch], or nullptr: one segment per sequence
  float* seg_decay;             // [n][heads][pitch]: base-2 logarithm of the segment's total decay per channel
};

template <int DP, int NV, bool STATE_ONLY>
struct ChannelShape {
  static constexpr int kPitch = DP + 8, kTile = kCTokens * kPitch;         // bf16 elements
  static constexpr int kVPitch = 64 * NV + 8, kVTile = kCTokens * kVPitch;
  static constexpr int kTiles = STATE_ONLY ? 2 : 10;
  static constexpr int kBuffer = (kTiles * kTile + kVTile) * 2 + (DP + 64) * 4;      // bytes: tiles, V, chunk decay, bonus parts
  static constexpr int kBuffers = DP <= 64 ? 2 : 1;
  static constexpr int kBytes = kBuffer * kBuffers;
};

template <int N>
__device__ __forceinline__ float row_shift(float v) {      // the lane N places in front inside the row of 16; 0 where there is none
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x110 | N, 0xf, 0xf, true));
}
template <int N>
__device__ __forceinline__ float row_lane(float v) {       // lane N of the row of 16
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x150 | N, 0xf, 0xf, true));
}

// N bf16 values as hi + lo at consecutive places of two tiles.
template <int N>
__device__ __forceinline__ void store_split(uint16_t* hi, uint16_t* lo, const float (&v)[N]) {
  uint32_t h[N / 2], l[N / 2];
#pragma unroll
  for (int e = 0; e < N / 2; ++e) {
    h[e] = pack_bf16x2(v[2 * e], v[2 * e + 1]);
    l[e] = pack_bf16x2(v[2 * e] - bf16lo_to_f32(h[e]), v[2 * e + 1] - bf16hi_to_f32(h[e]));
  }
  if (N == 2) {
    *reinterpret_cast<uint32_t*>(hi) = h[0];
    *reinterpret_cast<uint32_t*>(lo) = l[0];
  } else if (N == 4) {
    *reinterpret_cast<u32x2*>(hi) = u32x2{h[0], h[N / 2 - 1]};
    *reinterpret_cast<u32x2*>(lo) = u32x2{l[0], l[N / 2 - 1]};
  } else {
#pragma unroll
    for (int i = 0; i < N / 8; ++i) {
      store16(hi + 8 * i, u32x4{h[4 * i], h[(4 * i + 1) % (N / 2)], h[(4 * i + 2) % (N / 2)], h[(4 * i + 3) % (N / 2)]});
      store16(lo + 8 * i, u32x4{l[4 * i], l[(4 * i + 1) % (N / 2)], l[(4 * i + 2) % (N / 2)], l[(4 * i + 3) % (N / 2)]});
    }
  }
}

template <int DP, int NV, bool STATE_ONLY, bool VEC>
__global__ __launch_bounds__(256, DP <= 64 ? 3 : (DP <= 128 ? 2 : 1)) void channel_chunk_kernel(const ChannelArgs a) {
  using Sh = ChannelShape<DP, NV, STATE_ONLY>;
  constexpr int kC = DP / 16;                  // channels of a lane
  constexpr int kDT = DP / 16, kKS = DP / 32;  // 16-row pieces of the state, 32-deep steps
  constexpr int kVE = 4 * NV;                  // value elements a thread loads
  extern __shared__ __align__(16) unsigned char smem[];
  const int blocks = (a.vd + 64 * NV - 1) / (64 * NV);
  const int v0 = blockIdx.x % blocks * 64 * NV, h = blockIdx.x / blocks % a.heads, seg = blockIdx.x / blocks / a.heads;
  const int b = a.segments[3 * seg], t_begin = a.segments[3 * seg + 1], t_end = a.segments[3 * seg + 2];
  const int slot = a.state_slots[b], start = a.starts[b];
  if (slot < 0 || slot >= a.num_slots) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, n16 = lane & 15, jj = lane >> 4;
  const int vlen = a.vd - v0 < 64 * NV ? a.vd - v0 : 64 * NV;
  const int vx = wave * 16 * NV;               // this wave's first value column
  const bool active = vx < vlen;
  const int c0 = (4 * wave + jj) * kC;         // this lane's first channel in the first step
  const uint16_t *rp = a.r + (int64_t)h * a.d, *kp = a.k + (int64_t)h * a.d, *vp = a.v + (int64_t)h * a.vd + v0;
  const float* lp = a.log_decay + (int64_t)h * a.d;
  float u[kC], total[kC];
#pragma unroll
  for (int e = 0; e < kC; ++e) {
    u[e] = c0 + e < a.d ? a.bonus[(int64_t)h * a.d + c0 + e] : 0.f;
    total[e] = 0.f;
  }

  // S: tile (i, x), element e = row d = 16 i + 4 jj + e, column vx + 16 x + n16
  f32x4 st[kDT][NV];
  float* gstate = nullptr;
  bool load_state = false;
  if (!STATE_ONLY) {
    gstate = (a.seg_state ? a.seg_state + ((int64_t)seg * a.heads + h) * a.vd * a.pitch : a.state + ((int64_t)slot * a.heads + h) * a.vd * a.pitch) +
             (int64_t)v0 * a.pitch;
    load_state = a.seg_state || start > 0;
  }
#pragma unroll
  for (int i = 0; i < kDT; ++i)
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const int v = vx + 16 * x + n16, d = 16 * i + 4 * jj;
      const bool ok = load_state && v < vlen && d < a.pitch;
      st[i][x] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (!STATE_ONLY) {
        const f32x4 w = *reinterpret_cast<const f32x4*>(gstate + (ok ? (int64_t)v * a.pitch + d : 0));
#pragma unroll
        for (int e = 0; e < 4; ++e) st[i][x][e] = ok ? w[e] : 0.f;
      }
    }

  // ---- a chunk on its way: r, k and the decays of (token n16, channels c0..), values of (token tid / 16, columns (tid % 16) kVE ..)
  uint32_t r_raw[kC / 2], k_raw[kC / 2], v_raw[kVE / 2];
  float lw[kC];
  const int v_tok = threadIdx.x >> 4, v_col = (threadIdx.x & 15) * kVE;
  auto fetch = [&](int t0) {
    const int n = t_end - t0 < kCTokens ? t_end - t0 : kCTokens;
    const int64_t t = t0 + (n16 < n ? n16 : n - 1);
    if (VEC) {
      const int c = c0 < a.d ? c0 : 0;
      const uint16_t *rs = rp + t * a.r_stride + c, *ks = kp + t * a.k_stride + c;
      const float* ls = lp + t * a.decay_stride + c;
      if (kC == 2) {
        r_raw[0] = *reinterpret_cast<const uint32_t*>(rs);
        k_raw[0] = *reinterpret_cast<const uint32_t*>(ks);
        lw[0] = ls[0];
        lw[1] = ls[1];
      } else if (kC == 4) {
        const u32x2 x = *reinterpret_cast<const u32x2*>(rs), y = *reinterpret_cast<const u32x2*>(ks);
        const f32x4 z = *reinterpret_cast<const f32x4*>(ls);
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          r_raw[e % (kC / 2)] = x[e];
          k_raw[e % (kC / 2)] = y[e];
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) lw[e % kC] = z[e];
      } else {
#pragma unroll
        for (int i = 0; i < kC / 8; ++i) {
          const u32x4 x = load16(rs + 8 * i), y = load16(ks + 8 * i);
          const f32x4 z0 = *reinterpret_cast<const f32x4*>(ls + 8 * i), z1 = *reinterpret_cast<const f32x4*>(ls + 8 * i + 4);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            r_raw[(4 * i + e) % (kC / 2)] = x[e];
            k_raw[(4 * i + e) % (kC / 2)] = y[e];
            lw[(8 * i + e) % kC] = z0[e];
            lw[(8 * i + 4 + e) % kC] = z1[e];
          }
        }
      }
    } else {
#pragma unroll
      for (int e = 0; e < kC; ++e) {
        const int c = c0 + e < a.d ? c0 + e : 0;
        const uint32_t x = rp[t * a.r_stride + c], y = kp[t * a.k_stride + c];
        if (e & 1) {
          r_raw[e / 2] |= x << 16;
          k_raw[e / 2] |= y << 16;
        } else {
          r_raw[e / 2] = x;
          k_raw[e / 2] = y;
        }
        lw[e] = lp[t * a.decay_stride + c];
      }
    }
    const uint16_t* vs = vp + (int64_t)(t0 + (v_tok < n ? v_tok : n - 1)) * a.v_stride;
    if (VEC) {
      const int c = v_col < vlen ? v_col : 0;
      if (NV == 1) {
        const u32x2 x = *reinterpret_cast<const u32x2*>(vs + c);
        v_raw[0] = x[0];
        v_raw[1] = x[1];
      } else {
        const u32x4 x = load16(vs + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) v_raw[e % (kVE / 2)] = x[e];
      }
    } else {
#pragma unroll
      for (int e = 0; e < kVE; ++e) {
        const uint32_t x = v_col + e < vlen ? vs[v_col + e] : 0u;
        v_raw[e / 2] = e & 1 ? v_raw[e / 2] | x << 16 : x;
      }
    }
  };

  fetch(t_begin);
  int buf = 0;
  for (int t0 = t_begin; t0 < t_end; t0 += kCTokens, buf = Sh::kBuffers == 2 ? buf ^ 1 : 0) {
    const int n = t_end - t0 < kCTokens ? t_end - t0 : kCTokens;
    uint16_t* const tiles = reinterpret_cast<uint16_t*>(smem + buf * Sh::kBuffer);
    uint16_t* const ke_hi = tiles;
    uint16_t* const ke_lo = tiles + Sh::kTile;
    uint16_t* const rs_hi = tiles + 2 * Sh::kTile;      // not there in the states' pass
    uint16_t* const tv = tiles + Sh::kTiles * Sh::kTile;
    float* const chunk_decay = reinterpret_cast<float*>(tv + Sh::kVTile);
    float* const bonus_part = chunk_decay + DP;
    if (Sh::kBuffers == 1) __syncthreads();             // the last chunk's tiles have been read
    // ---- scaled rows
    {
      float rv[kC], kv[kC], L[kC], X[kC];
      const bool in = n16 < n;
      float direct = 0.f;
#pragma unroll
      for (int e = 0; e < kC; ++e) {
        const bool ok = in && c0 + e < a.d;
        rv[e] = ok ? (e & 1 ? bf16hi_to_f32(r_raw[e / 2]) : bf16lo_to_f32(r_raw[e / 2])) : 0.f;
        kv[e] = ok ? (e & 1 ? bf16hi_to_f32(k_raw[e / 2]) : bf16lo_to_f32(k_raw[e / 2])) : 0.f;
        float x = ok ? fmaxf(lw[e] * 1.4426950408889634f, kLeastLog2Decay) : 0.f;
        direct += rv[e] * u[e] * kv[e];
        x += row_shift<1>(x);
        x += row_shift<2>(x);
        x += row_shift<4>(x);
        x += row_shift<8>(x);
        L[e] = x;
        X[e] = row_shift<1>(x);
      }
      uint16_t* const row = tiles + n16 * Sh::kPitch + c0;
      float w[kC];
#pragma unroll
      for (int e = 0; e < kC; ++e) {
        const float end = row_lane<15>(L[e]);
        w[e] = kv[e] * __builtin_amdgcn_exp2f(end - L[e]);
        total[e] += end;
        if (n16 == 15) chunk_decay[c0 + e] = __builtin_amdgcn_exp2f(end);
      }
      store_split<kC>(row, row + Sh::kTile, w);
      if (!STATE_ONLY) {
#pragma unroll
        for (int e = 0; e < kC; ++e) w[e] = rv[e] * __builtin_amdgcn_exp2f(X[e]);
        store_split<kC>(row + 2 * Sh::kTile, row + 3 * Sh::kTile, w);
        float w2[kC];
#pragma unroll
        for (int e = 0; e < kC; ++e) {
          const float lo = row_lane<3>(L[e]), hi = row_lane<11>(L[e]);
          const float mid = n16 < 8 ? lo : hi;
          w[e] = rv[e] * __builtin_amdgcn_exp2f(X[e] - mid);
          w2[e] = kv[e] * __builtin_amdgcn_exp2f(mid - L[e]);
        }
        store_split<kC>(row + 4 * Sh::kTile, row + 5 * Sh::kTile, w);
        store_split<kC>(row + 6 * Sh::kTile, row + 7 * Sh::kTile, w2);
#pragma unroll
        for (int e = 0; e < kC; ++e) {
          const float border = row_lane<7>(L[e]);
          w[e] = (n16 < 8 ? kv[e] : rv[e]) * __builtin_amdgcn_exp2f(n16 < 8 ? border - L[e] : X[e] - border);
        }
        store_split<kC>(row + 8 * Sh::kTile, row + 9 * Sh::kTile, w);
        direct += __shfl_xor(direct, 16, kWave);
        direct += __shfl_xor(direct, 32, kWave);
        if (lane < 16) bonus_part[16 * wave + lane] = direct;
      }
      uint16_t* vd = tv + v_tok * Sh::kVPitch + v_col;
      if (NV == 1) *reinterpret_cast<u32x2*>(vd) = u32x2{v_raw[0], v_raw[1]};
      else store16(vd, u32x4{v_raw[0], v_raw[1], v_raw[2 % (kVE / 2)], v_raw[3 % (kVE / 2)]});
    }
    __syncthreads();
    if (t0 + kCTokens < t_end) fetch(t0 + kCTokens);
    if (!active) continue;

    // ---- products
    bf16x8 vb[NV];      // columns of V: tokens 4 jj .. 4 jj + 3, twice
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const s16x4 c = tile_block_columns(tv, Sh::kVPitch, 4 * jj, vx + 16 * x, lane);
      vb[x] = __builtin_bit_cast(bf16x8, join(c, c));
    }
    if (!STATE_ONLY) {
      f32x4 pd = {0.f, 0.f, 0.f, 0.f}, po = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < kKS; ++ks) {
        const int k0 = 32 * ks + 8 * jj;
        const bf16x8 rh = tile_row(tiles + 4 * Sh::kTile, Sh::kPitch, n16, k0), rl = tile_row(tiles + 5 * Sh::kTile, Sh::kPitch, n16, k0);
        const bf16x8 kh = tile_row(tiles + 6 * Sh::kTile, Sh::kPitch, n16, k0), kl = tile_row(tiles + 7 * Sh::kTile, Sh::kPitch, n16, k0);
        const bf16x8 bh = tile_row(tiles + 8 * Sh::kTile, Sh::kPitch, n16, k0), bl = tile_row(tiles + 9 * Sh::kTile, Sh::kPitch, n16, k0);
        pd = mfma16(kh, rh, pd);
        pd = mfma16(kh, rl, pd);
        pd = mfma16(kl, rh, pd);
        po = mfma16(bh, bh, po);
        po = mfma16(bh, bl, po);
        po = mfma16(bl, bh, po);
      }
      // O^T from the state
      f32x4 o[NV];
#pragma unroll
      for (int x = 0; x < NV; ++x) o[x] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < kKS; ++ks) {
        // the d's of a lane's eight values: 32 ks + 4 jj + 0..3 and 16 further on
        const uint16_t* q = rs_hi + n16 * Sh::kPitch + 32 * ks + 4 * jj;
        const u32x2 h0 = *reinterpret_cast<const u32x2*>(q), h1 = *reinterpret_cast<const u32x2*>(q + 16);
        const u32x2 l0 = *reinterpret_cast<const u32x2*>(q + Sh::kTile), l1 = *reinterpret_cast<const u32x2*>(q + Sh::kTile + 16);
        const bf16x8 qh = __builtin_bit_cast(bf16x8, u32x4{h0[0], h0[1], h1[0], h1[1]}), ql = __builtin_bit_cast(bf16x8, u32x4{l0[0], l0[1], l1[0], l1[1]});
#pragma unroll
        for (int x = 0; x < NV; ++x) {
          float s[8];
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            s[e] = st[2 * ks][x][e];
            s[4 + e] = st[2 * ks + 1][x][e];
          }
          bf16x8 hi, lo;
          split8(s, hi, lo);
          o[x] = mfma16(hi, qh, o[x]);
          o[x] = mfma16(hi, ql, o[x]);
          o[x] = mfma16(lo, qh, o[x]);
        }
      }
      // weights of token n16 on the tokens 4 jj .. 4 jj + 3
      const float own = (bonus_part[n16] + bonus_part[16 + n16]) + (bonus_part[32 + n16] + bonus_part[48 + n16]);
      float p[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int j = 4 * jj + e;
        const float below = n16 >= 8 && j < 8 ? po[e] : pd[e];
        p[e] = j < n16 ? below : (j == n16 ? own : 0.f);
      }
      u32x4 pw;
      pw[0] = pack_bf16x2(p[0], p[1]);
      pw[1] = pack_bf16x2(p[2], p[3]);
      pw[2] = pack_bf16x2(p[0] - bf16lo_to_f32(pw[0]), p[1] - bf16hi_to_f32(pw[0]));
      pw[3] = pack_bf16x2(p[2] - bf16lo_to_f32(pw[1]), p[3] - bf16hi_to_f32(pw[1]));
      const bf16x8 pb = __builtin_bit_cast(bf16x8, pw);
      uint16_t* orow = a.out + (int64_t)(t0 + n16) * a.out_stride + (int64_t)h * a.vd + v0 + vx + 4 * jj;
#pragma unroll
      for (int x = 0; x < NV; ++x) {
        o[x] = mfma16(vb[x], pb, o[x]);
        if (n16 < n) {
          if (VEC) {
            if (vx + 16 * x + 4 * jj < vlen) *reinterpret_cast<u32x2*>(orow + 16 * x) = u32x2{pack_bf16x2(o[x][0], o[x][1]), pack_bf16x2(o[x][2], o[x][3])};
          } else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
              if (vx + 16 * x + 4 * jj + e < vlen) orow[16 * x + e] = (uint16_t)f32_to_bf16_bits(o[x][e]);
          }
        }
      }
    }
    // S <- 2^{L_15} S + k^T V
#pragma unroll
    for (int i = 0; i < kDT; ++i) {
      const f32x4 w = *reinterpret_cast<const f32x4*>(chunk_decay + 16 * i + 4 * jj);
      const bf16x8 ka = __builtin_bit_cast(bf16x8, join(tile_block_columns(ke_hi, Sh::kPitch, 4 * jj, 16 * i, lane),
                                                        tile_block_columns(ke_lo, Sh::kPitch, 4 * jj, 16 * i, lane)));
#pragma unroll
      for (int x = 0; x < NV; ++x) {
#pragma unroll
        for (int e = 0; e < 4; ++e) st[i][x][e] *= w[e];
        st[i][x] = mfma16(ka, vb[x], st[i][x]);
      }
    }
  }

  float* dst = nullptr;
  if (STATE_ONLY) dst = a.seg_state + (((int64_t)seg * a.heads + h) * a.vd + v0) * a.pitch;
  else if (!a.seg_state) dst = gstate;
  if (dst && active) {
#pragma unroll
    for (int i = 0; i < kDT; ++i)
#pragma unroll
      for (int x = 0; x < NV; ++x) {
        const int v = vx + 16 * x + n16, d = 16 * i + 4 * jj;
        if (v < vlen && d < a.pitch) *reinterpret_cast<f32x4*>(dst + (int64_t)v * a.pitch + d) = st[i][x];
      }
  }
  if (STATE_ONLY && v0 == 0 && n16 == 0) {
#pragma unroll
    for (int e = 0; e < kC; ++e)
      if (c0 + e < a.pitch) a.seg_decay[((int64_t)seg * a.heads + h) * a.pitch + c0 + e] = total[e];
  }
}

// Start state of every segment (in place of its contribution) and the final state of every sequence.
__global__ __launch_bounds__(256) void channel_segment_scan_kernel(const ChannelArgs a, const int32_t* __restrict__ seq_segments) {
  const int h = blockIdx.y, b = blockIdx.z;
  const int64_t n = (int64_t)a.vd * a.pitch;
  const int64_t e = ((int64_t)blockIdx.x * 256 + threadIdx.x) * 4;
  const int slot = a.state_slots[b];
  if (e >= n || slot < 0 || slot >= a.num_slots) return;
  const int d = (int)(e % a.pitch);
  float* gs = a.state + ((int64_t)slot * a.heads + h) * n + e;
  f32x4 s = {0.f, 0.f, 0.f, 0.f};
  if (a.starts[b] > 0) s = *reinterpret_cast<const f32x4*>(gs);
  for (int seg = seq_segments[b]; seg < seq_segments[b + 1]; ++seg) {
    float* p = a.seg_state + ((int64_t)seg * a.heads + h) * n + e;
    const f32x4 u = *reinterpret_cast<const f32x4*>(p);
    const f32x4 l = *reinterpret_cast<const f32x4*>(a.seg_decay + ((int64_t)seg * a.heads + h) * a.pitch + d);
    *reinterpret_cast<f32x4*>(p) = s;
#pragma unroll
    for (int i = 0; i < 4; ++i) s[i] = __builtin_amdgcn_exp2f(l[i]) * s[i] + u[i];
  }
  *reinterpret_cast<f32x4*>(gs) = s;
}

static int columns_of(int64_t vd) { return vd <= 64 ? 64 : 128; }

template <int DP, int NV, bool VEC>
static int launch_channel(const ChannelArgs& a, const int32_t* seq_segments, int64_t batch, hipStream_t s) {
  using Full = ChannelShape<DP, NV, false>;
  using State = ChannelShape<DP, NV, true>;
  const int64_t items = (int64_t)a.num_segments * a.heads * ((a.vd + 64 * NV - 1) / (64 * NV));
  const dim3 grid((unsigned)items), block(256);
  static const hipError_t lds = hipFuncSetAttribute(reinterpret_cast<const void*>(&channel_chunk_kernel<DP, NV, false, VEC>),
                                                    hipFuncAttributeMaxDynamicSharedMemorySize, Full::kBytes);
  static const hipError_t lds_state = hipFuncSetAttribute(reinterpret_cast<const void*>(&channel_chunk_kernel<DP, NV, true, VEC>),
                                                          hipFuncAttributeMaxDynamicSharedMemorySize, State::kBytes);
  if (lds != hipSuccess) return record_hip_error(lds);
  if (lds_state != hipSuccess) return record_hip_error(lds_state);
  if (a.seg_state) {
    hipLaunchKernelGGL((channel_chunk_kernel<DP, NV, true, VEC>), grid, block, State::kBytes, s, a);
    const int64_t quads = ((int64_t)a.vd * a.pitch / 4 + 255) / 256;
    hipLaunchKernelGGL(channel_segment_scan_kernel, dim3((unsigned)quads, (unsigned)a.heads, (unsigned)batch), dim3(256), 0, s, a, seq_segments);
  }
  hipLaunchKernelGGL((channel_chunk_kernel<DP, NV, false, VEC>), grid, block, Full::kBytes, s, a);
  return finish_launch();
}

template <int NV, bool VEC>
static int launch_channel_for(const ChannelArgs& a, const int32_t* seq_segments, int64_t batch, hipStream_t s) {
  if (a.d <= 32) return launch_channel<32, NV, VEC>(a, seq_segments, batch, s);
  if (a.d <= 64) return launch_channel<64, NV, VEC>(a, seq_segments, batch, s);
  if (a.d <= 128) return launch_channel<128, NV, VEC>(a, seq_segments, batch, s);
  return launch_channel<256, NV, VEC>(a, seq_segments, batch, s);
}

}  // namespace mops

extern "C" int64_t mops_hip_channel_chunks_workgroups(int64_t heads, int64_t vd) {
  if (heads <= 0 || vd <= 0) return MOPS_HIP_EINVAL;
  return heads * ((vd + mops::columns_of(vd) - 1) / mops::columns_of(vd));
}

extern "C" int mops_hip_channel_chunks(const mops_hip_recurrence* r, const int32_t* segments, int64_t num_segments,
                                       const int32_t* seq_segments, float* seg_state, float* seg_decay, void* stream) {
  using namespace mops;
  if (!r || r->batch < 0 || num_segments < 0) return MOPS_HIP_EINVAL;
  if (r->batch == 0 || num_segments == 0) return MOPS_HIP_OK;
  if (r->dtype != MOPS_HIP_BF16 || r->conv_weight || r->rot || r->skip || r->k_scale != 1.f) return MOPS_HIP_EUNSUPPORTED;
  if (!r->q || !r->k || !r->v || !r->out || !r->state || !r->state_slots || !r->starts || !r->cu_seqlens || !segments) return MOPS_HIP_EINVAL;
  if (!r->channel_decay || !r->bonus || r->decay || r->dt) return MOPS_HIP_EINVAL;
  if (!seg_state != !seg_decay || (seg_state && !seq_segments) || (!seg_state && num_segments > r->batch)) return MOPS_HIP_EINVAL;
  if (r->heads <= 0 || r->groups != r->heads || r->d <= 0 || r->vd <= 0 || r->num_slots <= 0) return MOPS_HIP_EINVAL;
  if (r->d > 256 || r->heads > 65535 || r->batch > 65535 || r->vd > 65536) return MOPS_HIP_EUNSUPPORTED;
  if (r->q_stride < r->heads * r->d || r->k_stride < r->heads * r->d || r->v_stride < r->heads * r->vd || r->out_stride < r->heads * r->vd ||
      r->channel_decay_stride < r->heads * r->d)
    return MOPS_HIP_EINVAL;
  if (!aligned16(r->state) || (seg_state && (!aligned16(seg_state) || !aligned16(seg_decay)))) return MOPS_HIP_EALIGN;
  if (num_segments * r->heads * ((r->vd + 63) / 64) > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  ChannelArgs a;
  a.r = (const uint16_t*)r->q; a.k = (const uint16_t*)r->k; a.v = (const uint16_t*)r->v;
  a.log_decay = r->channel_decay; a.bonus = r->bonus;
  a.r_stride = r->q_stride; a.k_stride = r->k_stride; a.v_stride = r->v_stride; a.decay_stride = r->channel_decay_stride;
  a.out = (uint16_t*)r->out; a.out_stride = r->out_stride;
  a.state = r->state; a.num_slots = r->num_slots;
  a.state_slots = r->state_slots; a.cu_seqlens = r->cu_seqlens; a.starts = r->starts;
  a.segments = segments; a.num_segments = (int)num_segments;
  a.heads = (int)r->heads; a.d = (int)r->d; a.vd = (int)r->vd; a.pitch = (int)mops_hip_recurrence_state_pitch(r->d);
  a.seg_state = seg_state; a.seg_decay = seg_decay;
  const int64_t piece = r->d <= 128 ? 8 : 16;      // channels a lane may load at once
  const bool vec = r->d % piece == 0 && r->q_stride % 8 == 0 && r->k_stride % 8 == 0 && r->channel_decay_stride % 4 == 0 && aligned16(r->q) &&
                   aligned16(r->k) && aligned16(r->channel_decay) && r->vd % 8 == 0 && r->v_stride % 8 == 0 && r->out_stride % 8 == 0 &&
                   aligned16(r->v) && aligned16(r->out);
  hipStream_t s = (hipStream_t)stream;
  if (columns_of(r->vd) == 64) return vec ? launch_channel_for<1, true>(a, seq_segments, r->batch, s) : launch_channel_for<1, false>(a, seq_segments, r->batch, s);
  return vec ? launch_channel_for<2, true>(a, seq_segments, r->batch, s) : launch_channel_for<2, false>(a, seq_segments, r->batch, s);
}
