// The recurrence of decayed_recurrence.hip for portions of many tokens, 64 tokens at a time on the matrix cores (bf16 in,
// float32 accumulation and state):
//
//   L_i = sum of log a over the chunk up to token i,  s = input scale
//   O_i = e^{L_i} S^T q_i + sum_{j <= i} e^{L_i - L_j} s_j (q_i . k_j) v_j + skip v_i
//   S  <- e^{L_end} S + sum_j e^{L_end - L_j} s_j k_j v_j^T
//
// Workgroup (four waves) = (segment, NH heads of one q/k group, 128 / NH value columns of each), walking the chunks of its
// segment.  A wave owns 32 value columns of one head, with S [d x 32] in its accumulators from the first chunk to the last.
// All products are v_mfma_f32_32x32x16_bf16:
//   P^T [j, i] = K Q^T             one 32 x 32 tile per (head, tile below or on the diagonal), dealt out to the waves, weighted
//                                  and left in LDS for all of them
//   O^T [v, i] = S^T Q^T + V^T P^T S^T straight from the accumulators: their layout is an operand layout up to the order of the
//                                  d's inside a step, which Q's reads follow; V^T through transposing LDS reads
//   S [d, v]  += K^T (w V)         both operands through transposing LDS reads (ds_read_b64_tr_b16)
// What the recurrence keeps in 32 bits - the state, the decayed scores, the decayed values - enters a product as the sum of two
// bf16 numbers (value = hi + lo, 16 significant bits), at the price of a second MFMA.
//
// A matrix memory (MEMORY; decays and input scales per token from matrix_memory_gates_kernel) divides by its normalizer: n . q over the
// state in front of the chunk is a dot product per token on vector units, the rest are sums over the weighted scores.  n is the sum of
// four parts, one per wave and its sixteen tokens of every chunk.
//
// A sequence is one segment when there are enough sequences and heads to fill the chip.  Otherwise it is cut:
//   pass 1 (STATE_ONLY)  every segment from a zero state: its contribution and its total decay
//   pass 2 (scan)        the state at the start of every segment, and the final state into the sequence's slot
//   pass 3               every segment again, with outputs, from its start state
#include "matrix_memory.h"
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
  float k_scale, q_scale;       // of a matrix memory the one is 1, of the others the other
  const float *log_keep, *input_scale, *least;      // [tokens][heads]
  int copies;                   // rows of a head's state behind its values: copies of the normalizer, one per 64 values
  float* seg_state;             // [n][heads][vd + copies][pitch], or nullptr: one segment per sequence
  float* seg_decay;             // [n][heads]: base-2 logarithm of the segment's total decay
};

constexpr int kColumns = 128, kVPitch = kColumns + 8;     // value columns of a workgroup
constexpr int kPPitch = 32 + 8, kPTile = 32 * kPPitch;     // a weighted score tile [i][j]

template <int DP, int NH>
struct ChunkShape {
  static constexpr int kPitch = DP + 8;                    // elements; keeps 16-byte rows off each other's banks
  static constexpr int kK = kChunk * kPitch, kV = kChunk * kVPitch;
  static constexpr int kP = NH * 3 * 2 * kPTile;           // hi and lo of three tiles per head; takes the place of Q
  static constexpr int kQP = kK > kP ? kK : kP;
  // floats of a matrix memory behind the tables: least [64], n . q [64], sums of weighted scores [3][32], n [DP], its parts [4][DP]
  static constexpr int kMemory = 2 * kChunk + 96 + 5 * DP;
  static constexpr int bytes(bool state_only, bool memory) {
    return (kK + kV + (state_only ? 0 : kQP)) * 2 + (NH * (3 * kChunk + 32) + (memory ? kMemory : 0)) * 4;
  }
};

// q, k and v rows of a chunk on their way from memory into the LDS tiles: q and k rotated, scaled and rounded to bf16, zeros
// behind the head.  fetch() issues every load of a chunk at once, so that it can be called while the chunk
// before is still being worked on; store() finishes the values and writes the tiles.
// A thread owns pairs of 16-byte pieces of a row, for q and k alike: pair p < rot / 16 is columns (8p, 8p + rot/2), which
// rotate with each other; the pairs behind take two pieces that pass unchanged.
// ROT: rotation is compiled in (the tables take 16 registers a pair).
template <int DP, bool STATE_ONLY, int PAIRS, bool ROT>
struct ChunkLoader {
  static constexpr int kThreads = 256, kPitch = DP + 8;
  static constexpr int kVPieces = kChunk * (kColumns / 8) / kThreads;
  u32x4 k[PAIRS][2], q[STATE_ONLY ? 1 : PAIRS][2], v[kVPieces];
  f32x4 cs[ROT ? PAIRS : 1][2], sn[ROT ? PAIRS : 1][2];

  static __device__ __forceinline__ bool place(int i, const ChunkArgs& a, int& r, int& c0, int& c1, bool& rotates) {
    r = i / (DP / 16);
    const int p = i % (DP / 16), half = a.rot >> 1;
    rotates = ROT && 8 * p < half;
    c0 = rotates ? 8 * p : 16 * p;       // behind the rotated pairs: rot + 16 (p - rot / 16) = 16 p
    c1 = rotates ? c0 + half : c0 + 8;
    return i < kChunk * (DP / 16);
  }
  // Loads carry no condition: a row behind the chunk's end is the last row again (its input scale is zero, so it has no
  // weight anywhere), a column behind the head is column 0 and is dropped when the tile is written or by whoever reads the
  // tile.  Addresses are a uniform base and a 32-bit offset.
  static __device__ __forceinline__ u32x4 at(const void* base, uint32_t bytes) { return load16(static_cast<const char*>(base) + bytes); }
  __device__ __forceinline__ void fetch_qk(int first, const uint16_t* kp, const uint16_t* qp, int n, const ChunkArgs& a) {
#pragma unroll
    for (int j = 0; j < PAIRS; ++j) {
      int r, c0, c1;
      bool rotates;
      place((first + j) * kThreads + (int)threadIdx.x, a, r, c0, c1, rotates);
      r = r < n ? r : n - 1;
      c0 = c0 < a.d ? c0 : 0;
      c1 = c1 < a.d ? c1 : 0;
      const uint32_t kr = (uint32_t)r * (uint32_t)a.k_stride, qr = (uint32_t)r * (uint32_t)a.q_stride;
      k[j][0] = at(kp, 2 * (kr + c0));
      k[j][1] = at(kp, 2 * (kr + c1));
      if (!STATE_ONLY) {
        q[j][0] = at(qp, 2 * (qr + c0));
        q[j][1] = at(qp, 2 * (qr + c1));
      }
    }
  }
  __device__ __forceinline__ void fetch_trig(int first, int n, int pos0, const ChunkArgs& a) {
    if (!ROT || a.rot == 0) return;
#pragma unroll
    for (int j = 0; j < PAIRS; ++j) {
      int r, c0, c1;
      bool rotates;
      place((first + j) * kThreads + (int)threadIdx.x, a, r, c0, c1, rotates);
      r = pos0 + (r < n ? r : n - 1);
      r = r < (int)a.max_positions ? r : (int)a.max_positions - 1;
      const uint32_t from = 4 * ((uint32_t)r * (uint32_t)a.rot + (rotates ? c0 : 0));
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        cs[j][i] = __builtin_bit_cast(f32x4, at(a.cos_sin, from + 16 * i));
        sn[j][i] = __builtin_bit_cast(f32x4, at(a.cos_sin, from + 2 * a.rot + 16 * i));
      }
    }
  }
  // vp: the first head's columns; column c of the tile is value column (c % span) of head c / span
  __device__ __forceinline__ void fetch_v(const uint16_t* vp, int n, int span, int vlen, const ChunkArgs& a) {
#pragma unroll
    for (int j = 0; j < kVPieces; ++j) {
      const int i = j * kThreads + (int)threadIdx.x, r = i / (kColumns / 8), c = (i % (kColumns / 8)) * 8;
      const int x = c % span, head = c / span;
      v[j] = at(vp, 2 * ((uint32_t)(r < n ? r : n - 1) * (uint32_t)a.v_stride + head * a.vd + (x < vlen ? x : 0)));
    }
  }
  __device__ __forceinline__ void finish(uint16_t* tile, int r, int c0, int c1, const u32x4 (&w)[2], int j, bool rotates, float scale,
                                         const ChunkArgs& a) const {
    u32x4 o0 = w[0], o1 = w[1];
    if (ROT || scale != 1.f) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float x0 = bf16lo_to_f32(w[0][e]) * scale, x1 = bf16hi_to_f32(w[0][e]) * scale;
        const float y0 = bf16lo_to_f32(w[1][e]) * scale, y1 = bf16hi_to_f32(w[1][e]) * scale;
        if (ROT) {
          const int jj = ROT ? j : 0;
          const float ca = rotates ? cs[jj][e >> 1][2 * (e & 1)] : 1.f, cb = rotates ? cs[jj][e >> 1][2 * (e & 1) + 1] : 1.f;
          const float sa = rotates ? sn[jj][e >> 1][2 * (e & 1)] : 0.f, sb = rotates ? sn[jj][e >> 1][2 * (e & 1) + 1] : 0.f;
          o0[e] = pack_bf16x2(x0 * ca - y0 * sa, x1 * cb - y1 * sb);
          o1[e] = pack_bf16x2(y0 * ca + x0 * sa, y1 * cb + x1 * sb);
        } else {
          o0[e] = pack_bf16x2(x0, x1);
          o1[e] = pack_bf16x2(y0, y1);
        }
      }
    }
    const u32x4 zero = {0u, 0u, 0u, 0u};
    store16(tile + r * kPitch + c0, c0 < a.d ? o0 : zero);
    store16(tile + r * kPitch + c1, c1 < a.d ? o1 : zero);
  }
  __device__ __forceinline__ void store_qk(int first, uint16_t* tk, uint16_t* tq, const ChunkArgs& a) const {
#pragma unroll
    for (int j = 0; j < PAIRS; ++j) {
      int r, c0, c1;
      bool rotates;
      if (!place((first + j) * kThreads + (int)threadIdx.x, a, r, c0, c1, rotates)) continue;
      finish(tk, r, c0, c1, k[j], j, rotates, a.k_scale, a);
      if (!STATE_ONLY) finish(tq, r, c0, c1, q[j], j, rotates, 1.f, a);
    }
  }
  __device__ __forceinline__ void store_v(uint16_t* tv) const {
#pragma unroll
    for (int j = 0; j < kVPieces; ++j) {
      const int i = j * kThreads + (int)threadIdx.x;
      store16(tv + i / (kColumns / 8) * kVPitch + (i % (kColumns / 8)) * 8, v[j]);
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

template <int DP, int NH, bool STATE_ONLY, bool VEC, bool MEMORY>
__global__ __launch_bounds__(256, DP <= 128 ? 2 : 1) void decayed_chunk_kernel(const ChunkArgs a) {
  using S = ChunkShape<DP, NH>;
  constexpr int kDTiles = DP / 32, kSpan = kColumns / NH, kTilesPerHead = kSpan / 32;
  constexpr int kItems = NH * 3, kMine = (kItems + 3) / 4;        // weighted score tiles of the workgroup, of a wave
  extern __shared__ __align__(16) unsigned char smem[];
  uint16_t* const tk = reinterpret_cast<uint16_t*>(smem);
  uint16_t* const tv = tk + S::kK;
  uint16_t* const tq = tv + S::kV;                                // Q, then the weighted scores
  float* const tables = reinterpret_cast<float*>(tq + (STATE_ONLY ? 0 : S::kQP));
  // per head: [64] L, [64] input scale, [64] scale * 2^(L_end - L), [32] scale * 2^(L_31 - L), logarithms to base 2
  auto table = [&](int head) { return tables + head * (3 * kChunk + 32); };
  float* const least = tables + NH * (3 * kChunk + 32);           // MEMORY
  float* const n_dot_q = least + kChunk;
  float* const weight_sums = n_dot_q + kChunk;
  float* const n_all = weight_sums + 96;
  float* const n_parts = n_all + DP;

  // consecutive workgroups go to different XCDs: give each XCD a contiguous run of items, so that the heads that read the
  // same q and k rows share an L2
  const int blocks = NH == 1 ? (a.vd + kColumns - 1) / kColumns : 1, head_sets = a.heads / NH;
  const int total = a.num_segments * head_sets * blocks;
  const int per_xcd = (total + 7) / 8;
  const int item = (blockIdx.x % 8) * per_xcd + blockIdx.x / 8;
  if (blockIdx.x / 8 >= per_xcd || item >= total) return;
  const int v0 = (item % blocks) * kColumns;
  const int h0 = (item / blocks) % head_sets * NH;
  const int seg = item / (blocks * head_sets);
  const int b = a.segments[3 * seg], t_begin = a.segments[3 * seg + 1], t_end = a.segments[3 * seg + 2];
  const int slot = a.state_slots[b], start = a.starts[b], seq_begin = a.cu_seqlens[b];
  if (slot < 0 || slot >= a.num_slots) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x / 64, col = lane & 31, hh = lane >> 5;
  const int my_head = wave / kTilesPerHead, h = h0 + my_head;     // this wave's columns: head h, v0 + vx .. vx + 31
  const int vx = (wave % kTilesPerHead) * 32;
  const int vlen = a.vd - v0 < kSpan ? a.vd - v0 : kSpan;
  const bool active = vx < vlen;
  const int g = h0 / (a.heads / a.groups);
  const uint16_t *qp = a.q + (int64_t)g * a.d, *kp = a.k + (int64_t)g * a.d, *vp = a.v + (int64_t)h0 * a.vd + v0;
  constexpr float kLog2e = 1.4426950408889634f;
  // wave w also looks after the decays of head h0 + w
  const int decay_head = h0 + (wave < NH ? wave : 0);
  const float la_const = a.log_decay ? a.log_decay[decay_head] * kLog2e : 0.f;
  const float dt_bias = a.dt ? a.dt_bias[decay_head] : 0.f, neg_a = a.dt ? a.neg_a[decay_head] * kLog2e : 0.f;
  const float skip = a.skip ? a.skip[h] : 0.f;

  const int rows = a.vd + (MEMORY ? a.copies : 0);

  // S: tile i, register 4 q + e = row d = 32 i + 8 q + 4 hh + e, column vx + (lane & 31)
  f32x16 st[kDTiles];
  const int v_col = vx + col;
  auto state_d = [&](int i, int q4) { return 32 * i + 8 * q4 + 4 * hh; };
  float* gstate = nullptr;
  bool load_state = false;
  if (!STATE_ONLY) {
    if (a.seg_state) {
      gstate = a.seg_state + (((int64_t)seg * a.heads + h) * rows + v0) * a.pitch;
      load_state = true;
    } else {
      gstate = a.state + (((int64_t)slot * a.heads + h) * rows + v0) * a.pitch;
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

  constexpr int kPairsAll = (kChunk * (DP / 16) + 255) / 256;
  constexpr bool kAhead = VEC && kPairsAll <= 2;          // a whole chunk fits the registers next to the accumulators
  constexpr int kPairs = kPairsAll <= 2 ? kPairsAll : 2;
  ChunkLoader<DP, STATE_ONLY, kPairs, NH == 1 && !MEMORY> ld;      // heads that rotate do not share keys
  uint32_t dt_next = 0;      // this lane's time step of the next chunk, raw
  float keep_next = 0.f, scale_next = 0.f, least_next = 0.f;      // MEMORY: the same
  constexpr int kNorm = (DP + 63) / 64;
  float nn[MEMORY ? kNorm : 1];      // this wave's part of the normalizer: channels lane + 64 j
  if (MEMORY) {
#pragma unroll
    for (int j = 0; j < kNorm; ++j) {
      const int c = lane + 64 * j;
      const bool ok = wave == 0 && load_state && c < a.pitch;
      nn[MEMORY ? j : 0] = ok ? gstate[(int64_t)(a.vd - v0 + v0 / 64) * a.pitch + c] : 0.f;
      if (c < DP) n_parts[wave * DP + c] = nn[MEMORY ? j : 0];
    }
  }
  auto fetch = [&](int t) {
    const int m = t_end - t < kChunk ? t_end - t : kChunk;
    ld.fetch_qk(0, kp + (int64_t)t * a.k_stride, qp + (int64_t)t * a.q_stride, m, a);
    ld.fetch_trig(0, m, start + (t - seq_begin), a);
    ld.fetch_v(vp + (int64_t)t * a.v_stride, m, kSpan, vlen, a);
  };
  auto fetch_dt = [&](int t) {
    const int64_t row = t + lane < t_end ? t + lane : t_end - 1;
    if (MEMORY) {
      if (wave == 0) {
        keep_next = a.log_keep[row * a.heads + h];
        scale_next = a.input_scale[row * a.heads + h];
        least_next = a.least[row * a.heads + h];
      }
    } else if (a.dt) {
      dt_next = a.dt[row * a.dt_stride + decay_head];
    }
  };
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
      ld.fetch_v(vp + (int64_t)t0 * a.v_stride, n, kSpan, vlen, a);
      ld.store_v(tv);
#pragma unroll 1
      for (int first = 0; first < kPairsAll; first += kPairs) {
        ld.fetch_qk(first, kp + (int64_t)t0 * a.k_stride, qp + (int64_t)t0 * a.q_stride, n, a);
        ld.fetch_trig(first, n, pos0, a);
        ld.store_qk(first, tk, tq, a);
      }
    } else {
      load_tile_scalar<DP, 256>(tk, kp + (int64_t)t0 * a.k_stride, a.k_stride, n, pos0, a, a.k_scale);
      if (!STATE_ONLY) load_tile_scalar<DP, 256>(tq, qp + (int64_t)t0 * a.q_stride, a.q_stride, n, pos0, a, 1.f);
#pragma unroll 1
      for (int i = threadIdx.x; i < kChunk * kColumns; i += 256) {
        const int r = i / kColumns, c = i % kColumns;
        tv[r * kVPitch + c] = r < n && c % kSpan < vlen ? vp[(int64_t)(t0 + r) * a.v_stride + (int64_t)(c / kSpan) * a.vd + c % kSpan] : (uint16_t)0;
      }
    }
    if (wave < NH) {     // decays of the chunk: lane = token
      float la = 0.f, s = 0.f, l;
      if (MEMORY || a.dt) {
        if (lane < n) {
          s = MEMORY ? scale_next : softplus_f32(bf16lo_to_f32(dt_next) + dt_bias);
          la = MEMORY ? keep_next * kLog2e : neg_a * s;
        }
        if (MEMORY) least[lane] = least_next;
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
      const float l_end = __shfl(l, 63, 64), l_mid = __shfl(l, 31, 64);
      float* t = table(wave);
      t[lane] = l;
      t[kChunk + lane] = s;
      t[2 * kChunk + lane] = s * __builtin_amdgcn_exp2f(l_end - l);
      if (lane < 32) t[3 * kChunk + lane] = s * __builtin_amdgcn_exp2f(l_mid - l);
    }
    if (MEMORY && !STATE_ONLY)
      for (int c = threadIdx.x; c < DP; c += 256) n_all[c] = (n_parts[c] + n_parts[DP + c]) + (n_parts[2 * DP + c] + n_parts[3 * DP + c]);
    __syncthreads();
    const float* const mine = table(my_head);
    const float l_end = mine[kChunk - 1];
    total_log += l_end;
    const bool more = t0 + kChunk < t_end;
    if (more) fetch_dt(t0 + kChunk);

    if (!STATE_ONLY) {
      // ---- weighted scores: item = 3 * head + tile, tile 0: tokens 0..31 on themselves, 1: 32..63 on 0..31, 2: 32..63 on themselves
      bf16x8 p_hi[kMine][2], p_lo[kMine][2];
#pragma unroll
      for (int m = 0; m < kMine; ++m) {
        const int it = wave + 4 * m;
        if (it < kItems) {
          const int tile = it % 3, i_tok = (tile ? 32 : 0) + col, j_base = tile == 2 ? 32 : 0;
          const float* t = table(it / 3);
          f32x16 p;
#pragma unroll
          for (int r = 0; r < 16; ++r) p[r] = 0.f;
#pragma unroll
          for (int kk = 0; kk < DP / 16; ++kk)
            p = mfma32(tile_row(tk, S::kPitch, j_base + col, 16 * kk + 8 * hh), tile_row(tq, S::kPitch, i_tok, 16 * kk + 8 * hh), p);
          const float l_i = t[i_tok];
          float sum = 0.f;
          const float e_mid = tile == 1 ? __builtin_amdgcn_exp2f(l_i - t[31]) : 0.f;
#pragma unroll
          for (int half = 0; half < 2; ++half) {
            float w[8];
#pragma unroll
            for (int q4 = 0; q4 < 2; ++q4) {
              const int j0 = j_base + 16 * half + 8 * q4 + 4 * hh;
              const f32x4 l_j = *reinterpret_cast<const f32x4*>(t + j0), s_j = *reinterpret_cast<const f32x4*>(t + kChunk + j0);
              const f32x4 m_j = *reinterpret_cast<const f32x4*>(t + 3 * kChunk + (tile == 1 ? j0 : 0));
#pragma unroll
              for (int e = 0; e < 4; ++e) {
                // below the diagonal tiles the weight is a product of one factor per token on either side of the tile border
                const float on = j0 + e <= i_tok ? s_j[e] * __builtin_amdgcn_exp2f(l_i - l_j[e]) : 0.f;
                w[4 * q4 + e] = p[8 * half + 4 * q4 + e] * (tile == 1 ? m_j[e] * e_mid : on);
                if (MEMORY) sum += w[4 * q4 + e];
              }
            }
            split8(w, p_hi[m][half], p_lo[m][half]);
          }
          if (MEMORY) {
            sum += __shfl_xor(sum, 32, kWave);
            if (hh == 0) weight_sums[32 * tile + col] = sum;
          }
        }
      }
      if (MEMORY) {      // four lanes per token
        const int tok = threadIdx.x >> 2, part = threadIdx.x & 3;
        float dot = 0.f;
#pragma unroll
        for (int j = 0; j < DP / 32; ++j) {
          const int c = 32 * j + 8 * part;
          const u32x4 qw = load16(tq + tok * S::kPitch + c);
          const f32x4 n0 = *reinterpret_cast<const f32x4*>(n_all + c), n1 = *reinterpret_cast<const f32x4*>(n_all + c + 4);
#pragma unroll
          for (int e = 0; e < 4; ++e)
            dot += (e & 1 ? bf16hi_to_f32(qw[e >> 1]) : bf16lo_to_f32(qw[e >> 1])) * n0[e] +
                   (e & 1 ? bf16hi_to_f32(qw[2 + (e >> 1)]) : bf16lo_to_f32(qw[2 + (e >> 1)])) * n1[e];
        }
        dot += __shfl_xor(dot, 1, kWave);
        dot += __shfl_xor(dot, 2, kWave);
        if (part == 0) n_dot_q[tok] = dot * __builtin_amdgcn_exp2f(mine[tok]);
      }
      __builtin_amdgcn_sched_barrier(0);
      // ---- O^T = S^T Q^T, decayed
      f32x16 o[2];
#pragma unroll
      for (int it = 0; it < 2; ++it)
#pragma unroll
        for (int r = 0; r < 16; ++r) o[it][r] = 0.f;
      if (active) {
#pragma unroll
        for (int i = 0; i < kDTiles; ++i)
#pragma unroll
          for (int half = 0; half < 2; ++half) {
            float x[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) x[e] = st[i][8 * half + e];
            bf16x8 hi, lo;
            split8(x, hi, lo);
            const int d0 = 32 * i + 16 * half + 4 * hh;      // the d's of x: d0 .. d0+3, d0+8 .. d0+11
#pragma unroll
            for (int it = 0; it < 2; ++it) {
              const uint16_t* qr = tq + (32 * it + col) * S::kPitch + d0;
              const u32x2 w0 = *reinterpret_cast<const u32x2*>(qr), w1 = *reinterpret_cast<const u32x2*>(qr + 8);
              const bf16x8 qb = __builtin_bit_cast(bf16x8, u32x4{w0[0], w0[1], w1[0], w1[1]});
              o[it] = mfma32(hi, qb, o[it]);
              o[it] = mfma32(lo, qb, o[it]);
            }
          }
#pragma unroll
        for (int it = 0; it < 2; ++it) o[it] *= __builtin_amdgcn_exp2f(mine[32 * it + col]);
      }
      __syncthreads();     // Q has been read: the scores take its place
#pragma unroll
      for (int m = 0; m < kMine; ++m) {
        const int it = wave + 4 * m;
        if (it < kItems) {
          uint16_t* dst = tq + it * 2 * kPTile + col * kPPitch + 4 * hh;
#pragma unroll
          for (int half = 0; half < 2; ++half) {
            const u32x4 hw = __builtin_bit_cast(u32x4, p_hi[m][half]), lw = __builtin_bit_cast(u32x4, p_lo[m][half]);
            *reinterpret_cast<u32x2*>(dst + 16 * half) = u32x2{hw[0], hw[1]};
            *reinterpret_cast<u32x2*>(dst + 16 * half + 8) = u32x2{hw[2], hw[3]};
            *reinterpret_cast<u32x2*>(dst + kPTile + 16 * half) = u32x2{lw[0], lw[1]};
            *reinterpret_cast<u32x2*>(dst + kPTile + 16 * half + 8) = u32x2{lw[2], lw[3]};
          }
        }
      }
      __syncthreads();
      if (active) {
        const uint16_t* ph = tq + my_head * 6 * kPTile;
#pragma unroll
        for (int jt = 0; jt < 2; ++jt)
#pragma unroll
          for (int ks = 0; ks < 2; ++ks) {
            const int j0 = 32 * jt + 16 * ks + 8 * hh;
            const bf16x8 va = __builtin_bit_cast(bf16x8, tile_columns(tv, kVPitch, j0, j0 + 4, 32 * wave, lane));
#pragma unroll
            for (int it = jt; it < 2; ++it) {
              const uint16_t* tile = ph + (it + jt) * 2 * kPTile;      // (0,0) -> 0, (1,0) -> 1, (1,1) -> 2
              o[it] = mfma32(va, tile_row(tile, kPPitch, col, 16 * ks + 8 * hh), o[it]);
              o[it] = mfma32(va, tile_row(tile + kPTile, kPPitch, col, 16 * ks + 8 * hh), o[it]);
            }
          }
#pragma unroll
        for (int it = 0; it < 2; ++it) {
          const int i_tok = 32 * it + col;
          if (MEMORY) {
            const float sum = it == 0 ? weight_sums[col] : weight_sums[32 + col] + weight_sums[64 + col];
            o[it] *= a.q_scale / (fmaxf(a.q_scale * fabsf(n_dot_q[i_tok] + sum), least[i_tok]) + kMemoryEps);
          }
          if (skip != 0.f) {
#pragma unroll
            for (int q4 = 0; q4 < 4; ++q4)
#pragma unroll
              for (int e = 0; e < 4; ++e) o[it][4 * q4 + e] += skip * bf16lo_to_f32(tv[i_tok * kVPitch + 32 * wave + 8 * q4 + 4 * hh + e]);
          }
          uint16_t* orow = a.out + (int64_t)(t0 + i_tok) * a.out_stride + (int64_t)h * a.vd + v0 + vx;
#pragma unroll
          for (int half = 0; half < 2; ++half) {
            // eight consecutive columns per lane: the lower half of the wave completes piece 2 half, the upper half 2 half + 1
            const u32x2 even = {pack_bf16x2(o[it][8 * half], o[it][8 * half + 1]), pack_bf16x2(o[it][8 * half + 2], o[it][8 * half + 3])};
            const u32x2 odd = {pack_bf16x2(o[it][8 * half + 4], o[it][8 * half + 5]), pack_bf16x2(o[it][8 * half + 6], o[it][8 * half + 7])};
            const u32x2 keep = hh ? odd : even, give = hh ? even : odd;
            const u32x2 got = {(uint32_t)__shfl_xor((int)give[0], 32, 64), (uint32_t)__shfl_xor((int)give[1], 32, 64)};
            const u32x4 w = hh ? u32x4{got[0], got[1], keep[0], keep[1]} : u32x4{keep[0], keep[1], got[0], got[1]};
            const int v = 16 * half + 8 * hh;
            if (i_tok < n) {
              if (VEC) {
                if (vx + v < vlen) store16(orow + v, w);
              } else {
#pragma unroll
                for (int e = 0; e < 8; ++e)
                  if (vx + v + e < vlen) orow[v + e] = (uint16_t)(w[e >> 1] >> (16 * (e & 1)));
              }
            }
          }
        }
      }
    }
    // the next chunk is on its way while the state takes this one in; not before: its registers are in use above
    __builtin_amdgcn_sched_barrier(0);
    if (kAhead && more) fetch(t0 + kChunk);
    // ---- S <- e^{L_end} S + K^T (w V)
    if (active) {
      const float e_end = __builtin_amdgcn_exp2f(l_end);
#pragma unroll
      for (int i = 0; i < kDTiles; ++i) st[i] *= e_end;
#pragma unroll
      for (int ks = 0; ks < kChunk / 16; ++ks) {
        const int j0 = 16 * ks + 8 * hh;
        const s16x8 raw = tile_columns(tv, kVPitch, j0, j0 + 4, 32 * wave, lane);
        const f32x4 w0 = *reinterpret_cast<const f32x4*>(mine + 2 * kChunk + j0), w1 = *reinterpret_cast<const f32x4*>(mine + 2 * kChunk + j0 + 4);
        float x[8];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          x[e] = bf16lo_to_f32((uint16_t)raw[e]) * w0[e];
          x[4 + e] = bf16lo_to_f32((uint16_t)raw[4 + e]) * w1[e];
        }
        bf16x8 hi, lo;
        split8(x, hi, lo);
#pragma unroll
        for (int i = 0; i < kDTiles; ++i) {
          const bf16x8 ka = __builtin_bit_cast(bf16x8, tile_columns(tk, S::kPitch, j0, j0 + 4, 32 * i, lane));
          st[i] = mfma32(ka, hi, st[i]);
          st[i] = mfma32(ka, lo, st[i]);
        }
      }
    }
    if (MEMORY) {
      const float e_end = __builtin_amdgcn_exp2f(l_end);
#pragma unroll
      for (int j = 0; j < kNorm; ++j) {
        const int c = lane + 64 * j;
        float sum = nn[MEMORY ? j : 0] * e_end;
        if (c < DP) {
#pragma unroll
          for (int i = 0; i < kChunk / 4; ++i) {
            const int tok = kChunk / 4 * wave + i;
            sum += mine[2 * kChunk + tok] * bf16lo_to_f32(tk[tok * S::kPitch + c]);
          }
          n_parts[wave * DP + c] = sum;
        }
        nn[MEMORY ? j : 0] = sum;
      }
    }
  }

  float* dst = nullptr;
  if (STATE_ONLY) dst = a.seg_state + (((int64_t)seg * a.heads + h) * rows + v0) * a.pitch;
  else if (!a.seg_state) dst = gstate;
  if (dst && active) {
#pragma unroll
    for (int i = 0; i < kDTiles; ++i)
#pragma unroll
      for (int q4 = 0; q4 < 4; ++q4)
        if (v_col < vlen && state_d(i, q4) < a.pitch)
          *reinterpret_cast<f32x4*>(dst + v_col * a.pitch + state_d(i, q4)) = f32x4{st[i][4 * q4], st[i][4 * q4 + 1], st[i][4 * q4 + 2], st[i][4 * q4 + 3]};
  }
  if (MEMORY && dst) {      // this workgroup's copies
    __syncthreads();
    for (int c = threadIdx.x; c < a.pitch; c += 256) {
      const float sum = (n_parts[c] + n_parts[DP + c]) + (n_parts[2 * DP + c] + n_parts[3 * DP + c]);
      for (int i = v0 / 64; i < v0 / 64 + kColumns / 64 && i < a.copies; ++i) dst[(int64_t)(a.vd - v0 + i) * a.pitch + c] = sum;
    }
  }
  if (STATE_ONLY && v0 == 0 && vx == 0 && lane == 0) a.seg_decay[(int64_t)seg * a.heads + h] = total_log;
}

// Start state of every segment (in place of its contribution) and the final state of every sequence.  Segments of a sequence
// are consecutive; seq_segments[b], seq_segments[b + 1] bound them.
__global__ __launch_bounds__(256) void decayed_segment_scan_kernel(const ChunkArgs a, const int32_t* __restrict__ seq_segments) {
  const int h = blockIdx.y, b = blockIdx.z;
  const int64_t n = (int64_t)(a.vd + a.copies) * a.pitch;
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

template <int DP, int NH, bool VEC, bool MEMORY>
static int launch_chunks(const ChunkArgs& a, const int32_t* seq_segments, int64_t batch, hipStream_t s) {
  using S = ChunkShape<DP, NH>;
  const int64_t items = (int64_t)a.num_segments * (a.heads / NH) * (NH == 1 ? (a.vd + kColumns - 1) / kColumns : 1);
  const dim3 grid((unsigned)((items + 7) / 8 * 8)), block(256);
  static const hipError_t lds = hipFuncSetAttribute(reinterpret_cast<const void*>(&decayed_chunk_kernel<DP, NH, false, VEC, MEMORY>),
                                                    hipFuncAttributeMaxDynamicSharedMemorySize, S::bytes(false, MEMORY));
  static const hipError_t lds_state = hipFuncSetAttribute(reinterpret_cast<const void*>(&decayed_chunk_kernel<DP, NH, true, VEC, MEMORY>),
                                                          hipFuncAttributeMaxDynamicSharedMemorySize, S::bytes(true, MEMORY));
  if (lds != hipSuccess) return record_hip_error(lds);
  if (lds_state != hipSuccess) return record_hip_error(lds_state);
  if (a.seg_state) {
    hipLaunchKernelGGL((decayed_chunk_kernel<DP, NH, true, VEC, MEMORY>), grid, block, S::bytes(true, MEMORY), s, a);
    const int64_t quads = ((int64_t)(a.vd + a.copies) * a.pitch / 4 + 255) / 256;
    hipLaunchKernelGGL(decayed_segment_scan_kernel, dim3((unsigned)quads, (unsigned)a.heads, (unsigned)batch), dim3(256), 0, s, a, seq_segments);
  }
  hipLaunchKernelGGL((decayed_chunk_kernel<DP, NH, false, VEC, MEMORY>), grid, block, S::bytes(false, MEMORY), s, a);
  return finish_launch();
}

template <int NH, bool MEMORY = false>
static int launch_chunks_for(const ChunkArgs& a, const int32_t* seq_segments, int64_t batch, bool vec, hipStream_t s) {
  if (!vec) return a.d <= 64 ? launch_chunks<64, NH, false, MEMORY>(a, seq_segments, batch, s) : launch_chunks<256, NH, false, MEMORY>(a, seq_segments, batch, s);
  if (a.d <= 32) return launch_chunks<32, NH, true, MEMORY>(a, seq_segments, batch, s);
  if (a.d <= 64) return launch_chunks<64, NH, true, MEMORY>(a, seq_segments, batch, s);
  if (a.d <= 128) return launch_chunks<128, NH, true, MEMORY>(a, seq_segments, batch, s);
  return launch_chunks<256, NH, true, MEMORY>(a, seq_segments, batch, s);
}

// Gates of a matrix memory over the tokens of every (sequence, head), one workgroup each: with m_t = max(f_t + m_(t-1), i_t) the logarithm
// of the decay f_t + m_(t-1) - m_t, the input scale exp(i_t - m_t) and exp(-m_t); files the last m in all copies.  m is a scan over pairs
// (sum of f, greatest i carried to the end), four tokens per thread at a time.
constexpr int kGateThreads = 1024;

__global__ __launch_bounds__(kGateThreads) void matrix_memory_gates_kernel(const mops_hip_recurrence r, int copies, float* __restrict__ log_keep,
                                                                           float* __restrict__ input_scale, float* __restrict__ least) {
  __shared__ float wave_sum[kGateThreads / kWave], wave_most[kGateThreads / kWave];
  const int heads = (int)r.heads, h = blockIdx.x % heads, b = blockIdx.x / heads, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int slot = r.state_slots[b];
  if (slot < 0 || slot >= r.num_slots) return;
  const int t_begin = r.cu_seqlens[b], t_end = r.cu_seqlens[b + 1];
  float* const top = r.top + ((int64_t)slot * heads + h) * copies;
  float m = r.starts[b] > 0 ? top[0] : 0.f;
  const float input_bias = r.input_bias[h], forget_bias = r.forget_bias[h];
  for (int t0 = t_begin; t0 < t_end; t0 += 4 * kGateThreads) {
    float f[4], in[4], sum = 0.f, most = -INFINITY;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int64_t t = t0 + 4 * tid + e;
      f[e] = 0.f;
      in[e] = -INFINITY;      // behind the end: changes nothing
      if (t < t_end) {
        in[e] = capped_gate(bf16lo_to_f32(((const uint16_t*)r.input_gate)[t * r.gate_stride + h]) + input_bias, r.gate_cap);
        f[e] = log_sigmoid(capped_gate(bf16lo_to_f32(((const uint16_t*)r.forget_gate)[t * r.gate_stride + h]) + forget_bias, r.gate_cap));
      }
      most = fmaxf(most + f[e], in[e]);
      sum += f[e];
    }
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const float sum_up = __shfl_up(sum, off, 64), most_up = __shfl_up(most, off, 64);
      if (lane >= off) {
        most = fmaxf(most_up + sum, most);
        sum += sum_up;
      }
    }
    if (lane == 63) {
      wave_sum[wave] = sum;
      wave_most[wave] = most;
    }
    __syncthreads();
    float start = m;      // the maximum in front of this wave's tokens, then in front of this thread's
    for (int w = 0; w < wave; ++w) start = fmaxf(start + wave_sum[w], wave_most[w]);
    for (int w = 0; w < kGateThreads / kWave; ++w) m = fmaxf(m + wave_sum[w], wave_most[w]);
    float before = fmaxf(start + __shfl_up(sum, 1, 64), __shfl_up(most, 1, 64));
    if (lane == 0) before = start;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float now = fmaxf(f[e] + before, in[e]);
      const int64_t at = (int64_t)(t0 + 4 * tid + e) * heads + h;
      if (t0 + 4 * tid + e < t_end) {
        log_keep[at] = f[e] + before - now;
        input_scale[at] = expf(in[e] - now);
        least[at] = expf(-now);
      }
      before = now;
    }
    __syncthreads();
  }
  if (t_end > t_begin)
    for (int i = tid; i < copies; i += kGateThreads) top[i] = m;
}

// Heads of one workgroup: as many of a q/k group as fill its 128 value columns.
static int heads_together(int64_t heads, int64_t groups, int64_t vd, bool rotates) {
  const int64_t per = heads / groups;
  if (rotates) return 1;
  return vd <= 32 && per % 4 == 0 ? 4 : (vd <= 64 && per % 2 == 0 ? 2 : 1);
}

}  // namespace mops

extern "C" int64_t mops_hip_decayed_chunks_workgroups(int64_t heads, int64_t groups, int64_t vd) {
  if (heads <= 0 || groups <= 0 || heads % groups || vd <= 0) return MOPS_HIP_EINVAL;
  const int64_t nh = mops::heads_together(heads, groups, vd, false);
  return heads / nh * (nh == 1 ? (vd + mops::kColumns - 1) / mops::kColumns : 1);
}

extern "C" int mops_hip_matrix_memory_gates(const mops_hip_recurrence* r, float* log_keep, float* input_scale, float* least, void* stream) {
  using namespace mops;
  if (!r || r->batch < 0) return MOPS_HIP_EINVAL;
  if (r->batch == 0) return MOPS_HIP_OK;
  if (r->dtype != MOPS_HIP_BF16) return MOPS_HIP_EUNSUPPORTED;
  if (!r->input_gate || !r->forget_gate || !r->input_bias || !r->forget_bias || !r->top || !r->state_slots || !r->starts || !r->cu_seqlens || !log_keep ||
      !input_scale || !least || !(r->gate_cap > 0.f) || r->heads <= 0 || r->vd <= 0 || r->gate_stride < r->heads || r->num_slots <= 0)
    return MOPS_HIP_EINVAL;
  if (r->batch * r->heads > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  hipLaunchKernelGGL(matrix_memory_gates_kernel, dim3((unsigned)(r->batch * r->heads)), dim3(kGateThreads), 0, (hipStream_t)stream, *r,
                     (int)mops_hip_matrix_memory_copies(r->vd), log_keep, input_scale, least);
  return finish_launch();
}

extern "C" int mops_hip_decayed_chunks(const mops_hip_recurrence* r, const int32_t* segments, int64_t num_segments,
                                       const int32_t* seq_segments, float* seg_state, float* seg_decay, void* stream) {
  using namespace mops;
  if (!r || r->batch < 0 || num_segments < 0) return MOPS_HIP_EINVAL;
  if (r->batch == 0 || num_segments == 0) return MOPS_HIP_OK;
  if (r->dtype != MOPS_HIP_BF16 || r->conv_weight || r->channel_decay) return MOPS_HIP_EUNSUPPORTED;
  if (!r->q || !r->k || !r->v || !r->out || !r->state || !r->state_slots || !r->starts || !r->cu_seqlens || !segments) return MOPS_HIP_EINVAL;
  if (!seg_state != !seg_decay || (seg_state && !seq_segments) || (!seg_state && num_segments > r->batch)) return MOPS_HIP_EINVAL;
  if (r->heads <= 0 || r->groups <= 0 || r->heads % r->groups || r->d <= 0 || r->vd <= 0 || r->num_slots <= 0) return MOPS_HIP_EINVAL;
  if (r->d > 256 || r->heads > 65535 || r->batch > 65535 || r->vd > 65536) return MOPS_HIP_EUNSUPPORTED;
  if (r->q_stride < r->groups * r->d || r->k_stride < r->groups * r->d || r->v_stride < r->heads * r->vd || r->out_stride < r->heads * r->vd)
    return MOPS_HIP_EINVAL;
  if ((r->log_decay != nullptr) + (r->dt != nullptr) + (r->log_keep != nullptr) != 1) return MOPS_HIP_EINVAL;
  if (r->log_keep && (!r->input_scale || !r->least || r->groups != r->heads || r->rot || r->skip)) return MOPS_HIP_EINVAL;
  if (r->dt && (!r->dt_bias || !r->neg_a || r->dt_stride < r->heads)) return MOPS_HIP_EINVAL;
  if (r->rot < 0 || (r->rot & 1) || r->rot > r->d || (r->rot && (!r->cos_sin || r->max_positions <= 0))) return MOPS_HIP_EINVAL;
  if (!aligned16(r->state) || (seg_state && !aligned16(seg_state))) return MOPS_HIP_EALIGN;
  // offsets inside a chunk and into the table are 32 bits
  if (r->q_stride > (1 << 24) || r->k_stride > (1 << 24) || r->v_stride > (1 << 24) || r->max_positions * r->rot > (1 << 29)) return MOPS_HIP_EUNSUPPORTED;
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
  a.rot = (int)r->rot; a.max_positions = r->max_positions;
  a.k_scale = r->log_keep ? 1.f : r->k_scale; a.q_scale = r->log_keep ? r->k_scale : 1.f;
  a.log_keep = r->log_keep; a.input_scale = r->input_scale; a.least = r->least;
  a.copies = r->log_keep ? (int)mops_hip_matrix_memory_copies(r->vd) : 0;
  a.seg_state = seg_state; a.seg_decay = seg_decay;
  const bool vec = r->d % 8 == 0 && r->q_stride % 8 == 0 && r->k_stride % 8 == 0 && aligned16(r->q) && aligned16(r->k) &&
                   (r->rot == 0 || (r->rot % 16 == 0 && aligned16(r->cos_sin))) && r->vd % 8 == 0 && r->v_stride % 8 == 0 &&
                   r->out_stride % 8 == 0 && aligned16(r->v) && aligned16(r->out);
  if (a.log_keep) return launch_chunks_for<1, true>(a, seq_segments, r->batch, vec, (hipStream_t)stream);
  switch (heads_together(r->heads, r->groups, r->vd, r->rot > 0)) {
    case 4: return launch_chunks_for<4>(a, seq_segments, r->batch, vec, (hipStream_t)stream);
    case 2: return launch_chunks_for<2>(a, seq_segments, r->batch, vec, (hipStream_t)stream);
    default: return launch_chunks_for<1>(a, seq_segments, r->batch, vec, (hipStream_t)stream);
  }
}
