// Causal attention with a distance bias for long portions (bf16), keys and values straight from the pages: the tokens of the
// portion itself were filed there first.
//
// Workgroup (four waves) = (128 query tokens, head); a wave takes 32 queries.  64-token tiles of K and V in LDS, the next tile in
// flight into registers; a thread looks its token's page up one tile ahead.  v_mfma_f32_32x32x16_bf16 throughout:
//   S^T [key, query] = K Q^T        the softmax runs over keys: in a lane and its partner in the other half
//   O^T [v, query]  += V^T P^T      V^T through transposing LDS reads, P from the accumulators of S^T as the sum of two bf16 numbers
// Key tiles of which no query of a workgroup sees anything are left out, and a wave leaves out those of which its queries see nothing.
#include "mfma_tiles.h"
#include "visible.h"

namespace mops {

constexpr int kPrefillKeys = 64;

struct BiasedPrefillArgs {
  mops_hip_biased_attention a;      // row_seq and context_lens unused
  const int32_t* tiles;             // [n][5]: first query row, queries, position of the first, block table row, tokens of the context
  bool vec_out;
};

// NK: 16-deep steps of the key (dim <= 16 NK), NV: 32-wide pieces of the value (vdim <= 32 NV)
template <int NK, int NV, ScoreKind KIND>
__global__ __launch_bounds__(256, NK <= 8 && NV <= 4 ? 2 : 1) void biased_prefill_kernel(const BiasedPrefillArgs p) {
  constexpr int kPitchK = NK * 16 + 8, kPitchV = NV * 32 + 8;
  constexpr int kLoadsK = NK / 2, kLoadsV = NV;      // 16-byte pieces of a thread: columns 8 (tid % 4) + 32 j of token tid / 4
  __shared__ __align__(16) uint16_t tk[kPrefillKeys * kPitchK];
  __shared__ __align__(16) uint16_t tv[kPrefillKeys * kPitchV];
  const mops_hip_biased_attention& a = p.a;
  const int heads = (int)a.heads, groups = (int)a.kv_heads, vdim = (int)a.vdim, bs = (int)a.block_size;
  const int dp = ((int)a.dim + 7) / 8 * 8, vp = (vdim + 7) / 8 * 8;
  const int h = blockIdx.x % heads, g = h / (heads / groups);
  const int32_t* t = p.tiles + 5 * (int64_t)(blockIdx.x / heads);
  const int q_begin = t[0], q_count = t[1], pos0 = t[2], keys = t[4];
  const int32_t* table = a.block_table + (int64_t)t[3] * a.block_table_stride;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 31, hh = lane >> 5;
  const int qi = 32 * wave + col;                       // this lane's query of the tile
  const bool q_ok = qi < q_count;
  const int pos = pos0 + qi;

  bf16x8 qb[NK];
  {
    const uint16_t* qr = (const uint16_t*)a.q + ((int64_t)(q_begin + (q_ok ? qi : 0)) * heads + h) * dp;
#pragma unroll
    for (int kk = 0; kk < NK; ++kk) {
      const int c = 16 * kk + 8 * hh;
      qb[kk] = __builtin_bit_cast(bf16x8, q_ok && c < dp ? load16(qr + c) : u32x4{0u, 0u, 0u, 0u});
    }
  }
  f32x16 o[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[i][r] = 0.f;
  const float sink = a.sinks ? a.sinks[h] * 1.4426950408889634f : -INFINITY;      // a token with a value of zeros
  float m_run = !needs_reference(KIND) ? 0.f : sink, l_run = a.sinks && hh == 0 ? __builtin_amdgcn_exp2f(sink - m_run) : 0.f;

  const int visible = pos0 + q_count < keys ? pos0 + q_count : keys;      // keys any query of the tile sees
  const int keep = (int)a.keep_first, pos_first = pos0 + 32 * wave;      // of the wave's queries
  const VisibleBlocks<kPrefillKeys> blocks(first_visible(a, pos0), keep);
  const int n_blocks = blocks.count(visible);
  const int lo = first_visible(a, pos), lo_first = first_visible(a, pos_first), lo_last = first_visible(a, pos_first + 31);
  const int krow = tid >> 2, kcol = (tid & 3) * 8;
  u32x4 kreg[kLoadsK], vreg[kLoadsV];
  int block_next = 0, j_next = krow, blk_next = krow / bs, in_blk = krow % bs;      // the token page_of looks up next
  auto page_of = [&]() {      // row of this thread's next token in the pages, -1 without one
    if (block_next++ == blocks.kept && blocks.first > blocks.kept) {
      j_next = kPrefillKeys * blocks.first + krow;
      blk_next = j_next / bs;
      in_blk = j_next % bs;
    }
    int64_t row = -1;
    if (j_next < visible && blk_next < a.max_blocks) {
      const int id = table[blk_next];
      if (id >= 0 && id < a.num_blocks) row = (int64_t)id * bs + in_blk;
    }
    j_next += kPrefillKeys;
    in_blk += kPrefillKeys;
    while (in_blk >= bs) {
      in_blk -= bs;
      ++blk_next;
    }
    return row;
  };
  auto issue = [&](int64_t row) {
    const uint16_t *ks = (const uint16_t*)a.k_pages + ((row < 0 ? 0 : row) * groups + g) * dp;
    const uint16_t *vs = (const uint16_t*)a.v_pages + ((row < 0 ? 0 : row) * groups + g) * vp;
#pragma unroll
    for (int j = 0; j < kLoadsK; ++j) kreg[j] = load16(ks + (kcol + 32 * j < dp ? kcol + 32 * j : 0));      // columns behind the key meet zeros of the query
#pragma unroll
    for (int j = 0; j < kLoadsV; ++j) {
      vreg[j] = load16(vs + (kcol + 32 * j < vp ? kcol + 32 * j : 0));
      if (row < 0) vreg[j] = u32x4{0u, 0u, 0u, 0u};      // zero weights times what a page holds must be zero
    }
  };
  const ScoreOf<KIND> score(a, h);
  issue(page_of());
  int64_t next_row = page_of();
  for (int block = 0; block < n_blocks; ++block) {
    const int k0 = blocks.token(block);
    __syncthreads();
#pragma unroll
    for (int j = 0; j < kLoadsK; ++j) store16(tk + krow * kPitchK + kcol + 32 * j, kreg[j]);
#pragma unroll
    for (int j = 0; j < kLoadsV; ++j) store16(tv + krow * kPitchV + kcol + 32 * j, vreg[j]);
    __syncthreads();
    if (block + 1 < n_blocks) {
      issue(next_row);
      next_row = page_of();
    }
    if (k0 > pos_first + 31 || (k0 >= keep && k0 + kPrefillKeys <= lo_first)) continue;      // this wave's queries see none of the tile
    f32x16 s[2];
#pragma unroll
    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
      for (int r = 0; r < 16; ++r) s[kt][r] = 0.f;
#pragma unroll
    for (int kk = 0; kk < NK; ++kk)
#pragma unroll
      for (int kt = 0; kt < 2; ++kt) s[kt] = mfma32(tile_row(tk, kPitchK, 32 * kt + col, 16 * kk + 8 * hh), qb[kk], s[kt]);
    float m_loc = -INFINITY;
    const int last = pos < keys - 1 ? pos : keys - 1;
    const float dist = (float)(k0 + 4 * hh - pos);      // of the lane's first key, in front of the query by its negative
    // the diagonal, the end of the context or of what is visible: mask
    if (k0 + kPrefillKeys - 1 > pos_first || k0 + kPrefillKeys > keys || (k0 < lo_last && k0 + kPrefillKeys > keep)) {
#pragma unroll
      for (int kt = 0; kt < 2; ++kt)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int off = 32 * kt + 8 * (r >> 2) + (r & 3);
          const int j = k0 + 4 * hh + off;
          const float x = score(s[kt][r], dist + (float)off);
          s[kt][r] = j <= last && (j >= lo || j < keep) ? x : -INFINITY;
          m_loc = fmaxf(m_loc, s[kt][r]);
        }
    } else {
#pragma unroll
      for (int kt = 0; kt < 2; ++kt)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int off = 32 * kt + 8 * (r >> 2) + (r & 3);
          s[kt][r] = score(s[kt][r], dist + (float)off);
          m_loc = fmaxf(m_loc, s[kt][r]);
        }
    }
    float m_safe = 0.f;
    if (needs_reference(KIND)) {
      m_loc = fmaxf(m_loc, __shfl_xor(m_loc, 32, kWave));
      const float m_new = fmaxf(m_run, m_loc);
      m_safe = m_new == -INFINITY ? 0.f : m_new;
      const float alpha = __builtin_amdgcn_exp2f(m_run - m_safe);
      m_run = m_new;
      if (__any(alpha != 1.0f)) {
        l_run *= alpha;
#pragma unroll
        for (int i = 0; i < NV; ++i) o[i] *= alpha;
      }
    }
#pragma unroll
    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        float pv[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          pv[e] = score.weight(s[kt][8 * ks + e], m_safe);
          l_run += pv[e];
        }
        bf16x8 hi, lo;
        split8(pv, hi, lo);
        __builtin_amdgcn_sched_barrier(0);      // keeps the operand reads of the next step out of this one's registers
        const int j0 = 32 * kt + 16 * ks + 4 * hh;      // the keys of these eight values: j0 .. j0+3 and j0+8 .. j0+11
#pragma unroll
        for (int i = 0; i < NV; ++i) {
          const bf16x8 va = __builtin_bit_cast(bf16x8, tile_columns(tv, kPitchV, j0, j0 + 8, 32 * i, lane));
          o[i] = mfma32(va, hi, o[i]);
          o[i] = mfma32(va, lo, o[i]);
        }
      }
  }
  if (!q_ok) return;
  const float l = l_run + __shfl_xor(l_run, 32, kWave);
  const OutputGate<bf16_t> gate(a, q_begin + qi, h);
  const float inv = (KIND == kSigmoid ? 1.0f : (l > 0.f ? 1.0f / l : 0.f)) * (gate.each ? 1.0f : gate.constant);
  uint16_t* orow = (uint16_t*)a.out + (int64_t)(q_begin + qi) * a.out_stride + (int64_t)h * vdim;
#pragma unroll
  for (int i = 0; i < NV; ++i)
#pragma unroll
    for (int q4 = 0; q4 < 4; ++q4) {
      const int v = 32 * i + 8 * q4 + 4 * hh;
      float y[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) y[e] = o[i][4 * q4 + e] * inv;
      if (p.vec_out && v + 4 <= vdim) {
        if (gate.each) {
          const u32x2 g = *reinterpret_cast<const u32x2*>(gate.g + v);
#pragma unroll
          for (int e = 0; e < 4; ++e) y[e] *= gate.constant * sigmoid_for<bf16_t>(e & 1 ? bf16hi_to_f32(g[e >> 1]) : bf16lo_to_f32(g[e >> 1]));
        }
        *reinterpret_cast<u32x2*>(orow + v) = u32x2{pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3])};
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (v + e < vdim) orow[v + e] = (uint16_t)f32_to_bf16_bits(gate.each ? y[e] * gate(v + e) : y[e]);
      }
    }
}

int check_biased_attention(const mops_hip_biased_attention* a);   // biased_attention.hip

template <ScoreKind KIND>
static void launch_prefill(const BiasedPrefillArgs& p, dim3 grid, hipStream_t s) {
#define MOPS_BP(K, V) hipLaunchKernelGGL((biased_prefill_kernel<K, V, KIND>), grid, dim3(256), 0, s, p)
#define MOPS_BP_K(V) do { if (p.a.dim <= 64) MOPS_BP(4, V); else if (p.a.dim <= 128) MOPS_BP(8, V); else MOPS_BP(16, V); } while (0)
  if (p.a.vdim <= 64) MOPS_BP_K(2);
  else if (p.a.vdim <= 128) MOPS_BP_K(4);
  else MOPS_BP_K(8);
#undef MOPS_BP_K
#undef MOPS_BP
}

}  // namespace mops

extern "C" int mops_hip_biased_prefill(const mops_hip_biased_attention* args, const int32_t* tiles, int64_t num_tiles, void* stream) {
  using namespace mops;
  const int pre = check_biased_attention(args);
  if (pre != 1) return pre;
  if (num_tiles < 0 || (num_tiles && !tiles)) return MOPS_HIP_EINVAL;
  if (num_tiles == 0) return MOPS_HIP_OK;
  if (args->dtype != MOPS_HIP_BF16 || args->dim > 256 || args->vdim > 256 || num_tiles * args->heads > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  if (!aligned16(args->q) || !aligned16(args->k_pages) || !aligned16(args->v_pages)) return MOPS_HIP_EALIGN;
  BiasedPrefillArgs p;
  p.a = completed(*args);
  p.tiles = tiles;
  p.vec_out = args->vdim % 4 == 0 && p.a.out_stride % 4 == 0 && aligned16(args->out) &&
              (!args->gate || !args->gate_each || (args->gate_stride % 4 == 0 && aligned16(args->gate)));
  const dim3 grid((unsigned)(num_tiles * args->heads));
  hipStream_t s = (hipStream_t)stream;
  const ScoreKind kind = score_kind(*args);
  if (kind == kCappedFixed) launch_prefill<kCappedFixed>(p, grid, s);
  else if (kind == kCapped) launch_prefill<kCapped>(p, grid, s);
  else if (kind == kLogSloped) launch_prefill<kLogSloped>(p, grid, s);
  else if (kind == kSigmoid) launch_prefill<kSigmoid>(p, grid, s);
  else launch_prefill<kSloped>(p, grid, s);
  return finish_launch();
}
