// Query rows against paged keys and values on the matrix cores (bf16): the form of biased_attention_rows for decode steps and
// short portions.  HBM-bandwidth bound: all query heads of a group are served from one read of its keys and values.
//
// The 32-token stages of all rows are laid end to end and cut into equal runs, one per column of workgroups, whatever rows they
// belong to (every workgroup finds its run by a scan over the lengths; the host never reads them).  Workgroup = one wave = (column,
// kv head, up to 16 query heads of its group).  A stage is in flight from memory into registers while the one before is used out
// of the wave's LDS tiles.  v_mfma_f32_16x16x32_bf16:
//   S^T [token, head] = K Q^T
//   softmax over tokens, with the distance bias, in the layout the next product reads
//   O^T [v, head]    += V^T P^T      V^T through transposing LDS reads, P as the sum of two bf16 numbers
// A row that lies inside one run is written at once.  A row that is cut leaves (max, sum, unnormalised O) in one of the two slots
// of each run it touches; biased_combine_kernel merges them and writes the rows without any context as zeros.
// Weights that are sigmoids need no maximum and no sum; the parts of a cut row simply add up.
// Where rows see a part of their sequence only, their stages are those with something to see.  A sink enters with a row's first
// stage, as a token with a value of zeros.
#include "mfma_tiles.h"
#include "visible.h"

namespace mops {

constexpr int kStage = 32;
constexpr int kPlaneHeads = 16;
constexpr int kLeastStages = 2;      // shortest run

struct BiasedDecodeArgs {
  mops_hip_biased_attention a;
  int columns, head_tiles;
  int* plan;        // [0] stages per run, [1 + r] stages in front of row r, r <= rows
  float* part;      // [planes][columns][2][16][vdim]
  float* ml;        // [planes][columns][2][16][2]
};

// NK: 32-deep steps of the key (dim <= 32 NK); NV: 16-wide pieces of the value (vdim <= 16 NV)
template <int NK, int NV, ScoreKind KIND>
__global__ __launch_bounds__(64, NK * 32 + NV * 16 <= 256 ? 2 : 1) void biased_decode_kernel(const BiasedDecodeArgs p) {
  constexpr int kPitchK = 32 * NK + 8, kPitchV = 16 * NV + 8;
  constexpr int kPiecesK = 4 * NK, kPiecesV = 2 * NV;               // 16-byte pieces of a row
  constexpr int kLoadsK = kStage * kPiecesK / 64, kLoadsV = kStage * kPiecesV / 64;
  __shared__ __align__(16) uint16_t tk[kStage * kPitchK];
  __shared__ __align__(16) uint16_t tv[kStage * kPitchV];
  const mops_hip_biased_attention& a = p.a;
  const int groups = (int)a.kv_heads, planes = groups * p.head_tiles;
  const int plane = blockIdx.x % planes, column = blockIdx.x / planes;
  const int g = plane / p.head_tiles, ht = plane % p.head_tiles;
  const int heads = (int)a.heads, per_group = heads / groups, vdim = (int)a.vdim;
  const int dp = ((int)a.dim + 7) / 8 * 8, vp = (vdim + 7) / 8 * 8;
  const int lane = threadIdx.x, n = lane & 15, jj = lane >> 4;
  const bool head_ok = ht * kPlaneHeads + n < per_group;
  const int h = g * per_group + (head_ok ? ht * kPlaneHeads + n : 0);
  const int rows = (int)a.rows, bs = (int)a.block_size, max_tokens = (int)a.max_blocks * bs;
  auto length_of = [&](int r) {
    const int l = a.context_lens[r];
    return l < 0 ? 0 : (l < max_tokens ? l : max_tokens);
  };
  const int keep_first = (int)a.keep_first;
  auto blocks_of = [&](int len) { return VisibleBlocks<kStage>(visible_at(a, len).lo, keep_first); };
  auto stages_of = [&](int r) {
    const int len = length_of(r);
    return blocks_of(len).count(len);
  };

  // ---- this workgroup's run
  int row = 0, stage0 = 0, remaining;
  {
    const int share = (rows + 63) / 64, r0 = lane * share, r1 = r0 + share < rows ? r0 + share : rows;
    int sum = 0;
    for (int r = r0; r < r1; ++r) sum += stages_of(r);
    int incl = sum;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const int up = __shfl_up(incl, off, 64);
      if (lane >= off) incl += up;
    }
    const int front = incl - sum, total = __shfl(incl, 63, 64);
    int per = (total + p.columns - 1) / p.columns;
    if (per < kLeastStages) per = kLeastStages;
    if (blockIdx.x == 0) {      // for the combine kernel
      if (lane == 0) p.plan[0] = per;
      int at = front;
      for (int r = r0; r < r1; ++r) {
        p.plan[1 + r] = at;
        at += stages_of(r);
      }
      if (lane == 63) p.plan[1 + rows] = total;
    }
    const int64_t begin64 = (int64_t)column * per;
    if (begin64 >= total) return;
    const int begin = (int)begin64;
    remaining = total - begin < per ? total - begin : per;
    const bool mine = begin >= front && begin < front + sum;
    int r = r0, at = front;
    if (mine)
      for (int s = stages_of(r); begin >= at + s; s = stages_of(r)) {
        at += s;
        ++r;
      }
    const int owner = __ffsll((unsigned long long)__ballot(mine)) - 1;
    row = __builtin_amdgcn_readfirstlane(__shfl(r, owner, 64));
    stage0 = begin - __builtin_amdgcn_readfirstlane(__shfl(at, owner, 64));
  }

  // fixed places of this lane's pieces in a stage
  uint32_t k_off[kLoadsK], v_off[kLoadsV];
  int k_lds[kLoadsK], v_lds[kLoadsV];
#pragma unroll
  for (int j = 0; j < kLoadsK; ++j) {
    const int i = lane + 64 * j, t = i / kPiecesK, c = i % kPiecesK * 8;
    k_off[j] = (uint32_t)(t * groups * dp + (c < dp ? c : 0));      // columns behind the key meet zeros of the query
    k_lds[j] = t * kPitchK + c;
  }
#pragma unroll
  for (int j = 0; j < kLoadsV; ++j) {
    const int i = lane + 64 * j, t = i / kPiecesV, c = i % kPiecesV * 8;
    v_off[j] = (uint32_t)(t * groups * vp + (c < vp ? c : 0));      // columns behind the value are never stored
    v_lds[j] = t * kPitchV + c;
  }
  u32x4 kreg[kLoadsK], vreg[kLoadsV];
  const int32_t* table = nullptr;
  auto issue = [&](int tok0) {
    const int blk = tok0 / bs;
    const int id = blk < a.max_blocks ? __builtin_amdgcn_readfirstlane(table[blk]) : -1;
    const bool ok = id >= 0 && id < a.num_blocks;
    const int64_t t = (int64_t)(ok ? id : 0) * bs + tok0 % bs;
    const uint16_t *ks = (const uint16_t*)a.k_pages + (t * groups + g) * dp, *vs = (const uint16_t*)a.v_pages + (t * groups + g) * vp;
#pragma unroll
    for (int j = 0; j < kLoadsK; ++j) kreg[j] = load16_stream(ks + k_off[j]);
#pragma unroll
    for (int j = 0; j < kLoadsV; ++j) vreg[j] = load16_stream(vs + v_off[j]);
    return ok;
  };
  const ScoreOf<KIND> score(a, h);
  const float sink = a.sinks ? a.sinks[h] * 1.4426950408889634f : -INFINITY;

  for (; remaining > 0; ++row, stage0 = 0) {
    const int len = __builtin_amdgcn_readfirstlane(length_of(row));
    const Visible see = visible_at(a, len);
    const VisibleBlocks<kStage> blocks(see.lo, keep_first);
    const int row_stages = blocks.count(len);
    const int run = row_stages - stage0 < remaining ? row_stages - stage0 : remaining;
    if (run <= 0) continue;
    remaining -= run;
    table = a.block_table + (int64_t)(a.row_seq ? a.row_seq[row] : row) * a.block_table_stride;
    const uint16_t* q = (const uint16_t*)a.q + ((int64_t)row * heads + h) * dp;
    bf16x8 qb[NK];
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int c = 32 * i + 8 * jj;
      qb[i] = __builtin_bit_cast(bf16x8, head_ok && c < dp ? load16(q + c) : u32x4{0u, 0u, 0u, 0u});
    }
    bool ok_next = issue(blocks.token(stage0));
    f32x4 acc[NV];
#pragma unroll
    for (int i = 0; i < NV; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m_run = !needs_reference(KIND) ? 0.f : (stage0 == 0 ? sink : -INFINITY);
    float l_run = stage0 == 0 && jj == 0 && a.sinks ? __builtin_amdgcn_exp2f(sink - m_run) : 0.f;

    for (int st = stage0; st < stage0 + run; ++st) {
      const int tok0 = blocks.token(st);
      const int valid = ok_next ? (len - tok0 < kStage ? len - tok0 : kStage) : 0;
#pragma unroll
      for (int j = 0; j < kLoadsK; ++j) store16(tk + k_lds[j], kreg[j]);
#pragma unroll
      for (int j = 0; j < kLoadsV; ++j) store16(tv + v_lds[j], vreg[j]);
      if (valid < kStage) {      // rows behind the context: their weight is zero, and zero times what a page holds must be zero
#pragma unroll
        for (int j = 0; j < kLoadsV; ++j)
          if ((lane + 64 * j) / kPiecesV >= valid) store16(tv + v_lds[j], u32x4{0u, 0u, 0u, 0u});
      }
      if (st + 1 < stage0 + run) ok_next = issue(blocks.token(st + 1));
      __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
      __builtin_amdgcn_wave_barrier();
      __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
      f32x4 s[2];
#pragma unroll
      for (int tt = 0; tt < 2; ++tt) {
        s[tt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < NK; ++i) s[tt] = mfma16(tile_row(tk, kPitchK, 16 * tt + n, 32 * i + 8 * jj), qb[i], s[tt]);
      }
      float sv[8], m_loc = -INFINITY;
      const float dist = (float)(tok0 + 4 * jj - (len - 1));      // of the lane's first token, not positive for a valid one
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int t = 4 * jj + (e & 3) + 16 * (e >> 2);
        const float x = score(s[e >> 2][e & 3], dist + (float)((e & 3) + 16 * (e >> 2)));
        sv[e] = t < valid ? x : -INFINITY;
      }
      if (tok0 < see.lo && tok0 + kStage > see.kept) {      // the edge of what the row sees
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const int t = tok0 + 4 * jj + (e & 3) + 16 * (e >> 2);
          sv[e] = t >= see.lo || t < see.kept ? sv[e] : -INFINITY;
        }
      }
      float m_safe = 0.f, alpha = 1.f;
      if (needs_reference(KIND)) {
#pragma unroll
        for (int e = 0; e < 8; ++e) m_loc = fmaxf(m_loc, sv[e]);
        m_loc = fmaxf(m_loc, __shfl_xor(m_loc, 16, kWave));
        m_loc = fmaxf(m_loc, __shfl_xor(m_loc, 32, kWave));
        const float m_new = fmaxf(m_run, m_loc);
        m_safe = m_new == -INFINITY ? 0.f : m_new;
        alpha = __builtin_amdgcn_exp2f(m_run - m_safe);
        m_run = m_new;
      }
      float pv[8], psum = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        pv[e] = score.weight(sv[e], m_safe);
        psum += pv[e];
      }
      l_run = l_run * alpha + psum;
      if (needs_reference(KIND) && __any(alpha != 1.0f)) {
#pragma unroll
        for (int i = 0; i < NV; ++i) acc[i] *= alpha;
      }
      bf16x8 hi, lo;
      split8(pv, hi, lo);
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const bf16x8 va = __builtin_bit_cast(bf16x8, join(tile_block_columns(tv, kPitchV, 4 * jj, 16 * i, lane), tile_block_columns(tv, kPitchV, 16 + 4 * jj, 16 * i, lane)));
        acc[i] = mfma16(va, hi, acc[i]);
        acc[i] = mfma16(va, lo, acc[i]);
      }
      __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
      __builtin_amdgcn_wave_barrier();
      __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
    }
    float l_tot = l_run + __shfl_xor(l_run, 16, kWave);
    l_tot += __shfl_xor(l_tot, 32, kWave);
    if (!head_ok) continue;
    if (run == row_stages) {
      const float inv = KIND == kSigmoid ? 1.0f : (l_tot > 0.f ? 1.0f / l_tot : 0.f);
      const OutputGate<bf16_t> gate(a, row, h);
      uint16_t* orow = (uint16_t*)a.out + (int64_t)row * a.out_stride + (int64_t)h * vdim;
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int v = 16 * i + 4 * jj;
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (v + e < vdim) orow[v + e] = (uint16_t)f32_to_bf16_bits(acc[i][e] * inv * gate(v + e));
      }
      continue;
    }
    const int64_t slot = (((int64_t)plane * p.columns + column) * 2 + (stage0 > 0 ? 0 : 1)) * kPlaneHeads + n;
    float* prow = p.part + slot * vdim;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int v = 16 * i + 4 * jj;
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (v + e < vdim) prow[v + e] = acc[i][e];
    }
    if (jj == 0) {
      p.ml[2 * slot] = m_run;
      p.ml[2 * slot + 1] = l_tot;
    }
  }
}

// One wave per (row, head).
__global__ __launch_bounds__(64) void biased_combine_kernel(const BiasedDecodeArgs p) {
  const mops_hip_biased_attention& a = p.a;
  const int heads = (int)a.heads, vdim = (int)a.vdim, per_group = heads / (int)a.kv_heads;
  const int h = blockIdx.x % heads, row = blockIdx.x / heads, lane = threadIdx.x;
  const int per = p.plan[0], f0 = p.plan[1 + row], f1 = p.plan[2 + row];
  uint16_t* out = (uint16_t*)a.out + (int64_t)row * a.out_stride + (int64_t)h * vdim;
  if (f1 <= f0) {
    for (int v = lane; v < vdim; v += kWave) out[v] = 0;
    return;
  }
  const int j0 = f0 / per, j1 = (f1 - 1) / per;
  if (j0 == j1) return;
  const int plane = h / per_group * p.head_tiles + h % per_group / kPlaneHeads, n = h % per_group % kPlaneHeads;
  // slot 1 in the run where the row begins, slot 0 in the following ones
  auto slot_of = [&](int j) { return (((int64_t)plane * p.columns + j) * 2 + (j == j0 ? 1 : 0)) * kPlaneHeads + n; };
  float m = -INFINITY;
  for (int j = j0 + lane; j <= j1; j += kWave) m = fmaxf(m, p.ml[2 * slot_of(j)]);
  m = group_max<kWave>(m);
  const float safe = m == -INFINITY ? 0.f : m;
  float l = 0.f;
  for (int j = j0 + lane; j <= j1; j += kWave) l += __builtin_amdgcn_exp2f(p.ml[2 * slot_of(j)] - safe) * p.ml[2 * slot_of(j) + 1];
  l = group_sum<kWave>(l);
  const float inv = a.weight_bias ? 1.0f : (l > 0.f ? 1.0f / l : 0.f);
  const OutputGate<bf16_t> gate(a, row, h);
  for (int v0 = 0; v0 < vdim; v0 += 4 * kWave) {
    float o[4] = {0.f, 0.f, 0.f, 0.f};
    for (int j = j0; j <= j1; ++j) {
      const int64_t s = slot_of(j);
      const float w = __builtin_amdgcn_exp2f(p.ml[2 * s] - safe);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int v = v0 + e * kWave + lane;
        if (v < vdim) o[e] += w * p.part[s * vdim + v];
      }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int v = v0 + e * kWave + lane;
      if (v < vdim) out[v] = (uint16_t)f32_to_bf16_bits(o[e] * inv * gate(v));
    }
  }
}

int check_biased_attention(const mops_hip_biased_attention* a);   // biased_attention.hip

// Eight waves per CU of 256, fewer where the registers of a stage allow one wave per SIMD only.
static int decode_columns(int64_t dim, int64_t vdim, int64_t planes) {
  const int64_t waves = dim <= 64 && vdim <= 64 ? 4096 : (dim <= 128 && vdim <= 128 ? 2048 : 1024);
  const int64_t c = waves / planes;
  return c < 16 ? 16 : (int)c;
}
static int64_t decode_plan_bytes(int64_t rows) { return ((rows + 2) * 4 + 255) / 256 * 256; }
static int64_t head_tiles_of(int64_t heads, int64_t kv_heads) { return (heads / kv_heads + kPlaneHeads - 1) / kPlaneHeads; }

template <int NK, ScoreKind KIND>
static void launch_decode_keys(const BiasedDecodeArgs& p, dim3 grid, hipStream_t s) {
  const int64_t v = p.a.vdim;
  if (v <= 32) hipLaunchKernelGGL((biased_decode_kernel<NK, 2, KIND>), grid, dim3(64), 0, s, p);
  else if (v <= 64) hipLaunchKernelGGL((biased_decode_kernel<NK, 4, KIND>), grid, dim3(64), 0, s, p);
  else if (v <= 128) hipLaunchKernelGGL((biased_decode_kernel<NK, 8, KIND>), grid, dim3(64), 0, s, p);
  else hipLaunchKernelGGL((biased_decode_kernel<NK, 16, KIND>), grid, dim3(64), 0, s, p);
}
template <ScoreKind KIND>
static void launch_decode(const BiasedDecodeArgs& p, dim3 grid, hipStream_t s) {
  const int64_t d = p.a.dim;
  if (d <= 32) launch_decode_keys<1, KIND>(p, grid, s);
  else if (d <= 64) launch_decode_keys<2, KIND>(p, grid, s);
  else if (d <= 128) launch_decode_keys<4, KIND>(p, grid, s);
  else launch_decode_keys<8, KIND>(p, grid, s);
}

}  // namespace mops

extern "C" int64_t mops_hip_biased_decode_workspace_bytes(int64_t rows, int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim) {
  using namespace mops;
  if (rows <= 0 || heads <= 0 || kv_heads <= 0 || heads % kv_heads || dim <= 0 || vdim <= 0) return 0;
  const int64_t planes = kv_heads * head_tiles_of(heads, kv_heads);
  return decode_plan_bytes(rows) + planes * decode_columns(dim, vdim, planes) * 2 * kPlaneHeads * (vdim + 2) * (int64_t)sizeof(float);
}

extern "C" int mops_hip_biased_decode(const mops_hip_biased_attention* a, void* workspace, int64_t workspace_bytes, void* stream) {
  using namespace mops;
  const int pre = check_biased_attention(a);
  if (pre != 1) return pre;
  if (a->dtype != MOPS_HIP_BF16 || a->dim > 256 || a->vdim > 256 || a->block_size % kStage) return MOPS_HIP_EUNSUPPORTED;
  if (!aligned16(a->q) || !aligned16(a->k_pages) || !aligned16(a->v_pages)) return MOPS_HIP_EALIGN;
  const int64_t tokens = a->max_blocks * a->block_size;
  if (a->rows * ((tokens + kStage - 1) / kStage) > 0x7fffffffLL || a->kv_heads * 256 * kStage > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  BiasedDecodeArgs p;
  p.a = completed(*a);
  p.head_tiles = (int)head_tiles_of(a->heads, a->kv_heads);
  const int64_t planes = a->kv_heads * p.head_tiles;
  p.columns = decode_columns(a->dim, a->vdim, planes);
  if (planes * p.columns > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  if (!workspace || workspace_bytes < mops_hip_biased_decode_workspace_bytes(a->rows, a->heads, a->kv_heads, a->dim, a->vdim)) return MOPS_HIP_EWORKSPACE;
  if (!aligned16(workspace)) return MOPS_HIP_EALIGN;
  p.plan = (int*)workspace;
  p.part = (float*)((char*)workspace + decode_plan_bytes(a->rows));
  p.ml = p.part + planes * p.columns * 2 * kPlaneHeads * a->vdim;
  const dim3 grid((unsigned)(planes * p.columns));
  hipStream_t s = (hipStream_t)stream;
  const ScoreKind kind = score_kind(*a);
  if (kind == kCappedFixed) launch_decode<kCappedFixed>(p, grid, s);
  else if (kind == kCapped) launch_decode<kCapped>(p, grid, s);
  else if (kind == kLogSloped) launch_decode<kLogSloped>(p, grid, s);
  else if (kind == kSigmoid) launch_decode<kSigmoid>(p, grid, s);
  else launch_decode<kSloped>(p, grid, s);
  hipLaunchKernelGGL(biased_combine_kernel, dim3((unsigned)(a->rows * a->heads)), dim3(64), 0, s, p);
  return finish_launch();
}
