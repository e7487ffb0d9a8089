// Query rows against the paged latent cache on the matrix cores (bf16): the form of latent_attention_rows for decode steps
// and short portions.  The cache row is key and value at once, so it is read once per 16 heads.
//
// The 32-token tiles of all rows are laid end to end and cut into equal runs, one per workgroup and 16 heads, whatever rows
// they belong to, so that contexts of different lengths cost no imbalance (every workgroup finds its run by a scan over the
// lengths; the host never reads them).  Workgroup = four waves; the next tile is in flight into registers while this one is
// used out of LDS.
//   S^T [token, head] = C Q^T    a wave takes 16 tokens and every second 32-wide k step; the two partial sums meet in LDS
//   softmax over tokens          every wave, redundantly, in the layout the next product reads
//   O^T [r, head] += C^T P^T     a wave takes every fourth 16-wide piece of the latent; C^T through transposing LDS reads,
//                                P as the sum of two bf16 numbers
// A row that lies inside one run is written at once.  A row that is cut leaves (max, sum, unnormalised O) in one of the two
// slots of each run it touches; latent_combine_kernel merges them and writes the rows without any context as zeros.
#include "mfma_tiles.h"

namespace mops {

constexpr int kTileTokens = 32;
constexpr int kHeadTile = 16;

constexpr int kMinTiles = 4;     // shortest run: below, merging costs more than it saves

struct LatentDecodeArgs {
  mops_hip_latent_rows a;
  int columns, head_tiles;
  int* plan;        // [0] tiles per run, [1 + r] tiles in front of row r, r <= rows
  float* part;      // [head_tiles][columns][2][16][kv_rank]
  float* ml;        // [head_tiles][columns][2][16][2]
  bool vec_q;
};

// NQ: 32-wide k steps per wave (kv_rank + rot_dim <= 64 NQ); NT: 16-wide latent pieces per wave (kv_rank <= 64 NT)
template <int NQ, int NT>
__global__ __launch_bounds__(256, 2) void latent_decode_kernel(const LatentDecodeArgs p) {
  constexpr int kMaxPitch = 64 * NQ + 8;
  __shared__ __align__(16) uint16_t tile[kTileTokens * kMaxPitch];
  __shared__ __align__(16) float part_s[2][kTileTokens][kHeadTile + 1];
  __shared__ int s_scan[4], s_row, s_front;
  const mops_hip_latent_rows& a = p.a;
  const int column = blockIdx.x % p.columns, ht = blockIdx.x / p.columns;
  const int heads = (int)a.heads, kv_rank = (int)a.kv_rank, rot = (int)a.rot_dim, width = kv_rank + rot;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int n = lane & 15, jj = lane >> 4;
  const int h = ht * kHeadTile + n;
  const int rows = (int)a.rows, bs = (int)a.block_size, max_tokens = (int)a.max_blocks * bs;
  auto length_of = [&](int r) {
    const int n = a.context_lens[r];
    return n < 0 ? 0 : (n < max_tokens ? n : max_tokens);
  };
  auto tiles_of = [&](int r) { return (length_of(r) + kTileTokens - 1) / kTileTokens; };

  // ---- this workgroup's run
  int total, per;
  {
    const int share = (rows + 255) / 256, r0 = tid * share, r1 = r0 + share < rows ? r0 + share : rows;
    int sum = 0;
    for (int r = r0; r < r1; ++r) sum += tiles_of(r);
    int incl = sum;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const int up = __shfl_up(incl, off, 64);
      if (lane >= off) incl += up;
    }
    if (lane == 63) s_scan[wave] = incl;
    __syncthreads();
    int front = incl - sum;
    for (int w = 0; w < wave; ++w) front += s_scan[w];
    total = s_scan[0] + s_scan[1] + s_scan[2] + s_scan[3];
    per = (total + p.columns - 1) / p.columns;
    if (per < kMinTiles) per = kMinTiles;
    const int64_t begin = (int64_t)column * per;
    if (blockIdx.x == 0) {      // for the combine kernel
      if (tid == 0) p.plan[0] = per;
      int at = front;
      for (int r = r0; r < r1; ++r) {
        p.plan[1 + r] = at;
        at += tiles_of(r);
      }
      if (tid == 255) p.plan[1 + rows] = total;
    }
    if (begin >= total) return;
    if (begin >= front && begin < front + sum) {
      int r = r0, at = front;
      for (int n = tiles_of(r); begin >= at + n; n = tiles_of(r)) {
        at += n;
        ++r;
      }
      s_row = r;
      s_front = at;
    }
    __syncthreads();
  }
  int row = s_row, tile0 = column * per - s_front;
  int remaining = total - column * per < per ? total - column * per : per;

  const int ksteps = (width + 31) >> 5, lp = ksteps * 32 + 8, row_pieces = ksteps * 4;
  const int32_t* table = nullptr;
  int tok_end = 0;
  // this thread's pieces of a tile: fixed (token, column) pairs
  u32x4 reg[NQ];
  auto piece_row = [&](int j) { return (tid + 256 * j) / row_pieces; };
  auto piece_col = [&](int j) { return ((tid + 256 * j) % row_pieces) * 8; };
  int pr[NQ], pc[NQ];
#pragma unroll
  for (int j = 0; j < NQ; ++j) {
    pr[j] = piece_row(j);
    pc[j] = piece_col(j);
  }
  auto issue = [&](int tok0) {
    const int blk = tok0 / bs;
    const int id = blk < a.max_blocks ? table[blk] : -1;
    const bool ok = id >= 0 && id < a.num_blocks;
    const uint16_t* src = (const uint16_t*)a.cache + ((int64_t)(ok ? id : 0) * bs + tok0 % bs) * a.pitch;
#pragma unroll
    for (int j = 0; j < NQ; ++j) {
      reg[j] = u32x4{0u, 0u, 0u, 0u};
      if (ok && pr[j] < kTileTokens && tok0 + pr[j] < tok_end && pc[j] < a.pitch) reg[j] = load16_stream(src + pr[j] * a.pitch + pc[j]);
    }
    return ok;
  };
  const int tt = wave & 1, kh = wave >> 1;
  const float scale_log2 = a.scale * 1.4426950408889634f;

  for (; remaining > 0; ++row, tile0 = 0) {
    const int len = length_of(row), row_tiles = (len + kTileTokens - 1) / kTileTokens;
    const int run = row_tiles - tile0 < remaining ? row_tiles - tile0 : remaining;
    if (run <= 0) continue;
    remaining -= run;
    const int tok_begin = tile0 * kTileTokens;
    tok_end = tok_begin + run * kTileTokens < len ? tok_begin + run * kTileTokens : len;
    table = a.block_table + (int64_t)(a.row_seq ? a.row_seq[row] : row) * a.block_table_stride;
    bool ok_next = issue(tok_begin);
    __syncthreads();      // the last piece's tile has been read

    // ---- query rows [16 heads][k] through LDS into B operands: [latent | rotated part | zeros]
    {
      const int pos = len - 1;
      const float* trig = a.cos_sin + (int64_t)(pos < a.max_positions ? pos : a.max_positions - 1) * rot;
#pragma unroll 1
      for (int i = tid; i < kHeadTile * (lp >> 3); i += 256) {
        const int hr = i / (lp >> 3), c = (i % (lp >> 3)) * 8;
        const int head = ht * kHeadTile + hr;
        u32x4 w = {0u, 0u, 0u, 0u};
        if (head < heads && c < width) {
          const uint16_t* ql = (const uint16_t*)a.q_latent + ((int64_t)row * heads + head) * kv_rank;
          const uint16_t* qr = (const uint16_t*)a.q_rot + (int64_t)row * a.q_rot_token_stride + head * a.q_rot_head_stride;
          if (p.vec_q && c + 8 <= kv_rank) {
            w = load16(ql + c);
          } else if (p.vec_q) {       // four pairs of the rotated part
            const int d = c - kv_rank;
            const u32x4 raw = load16(qr + d);
            const f32x4 cs = *reinterpret_cast<const f32x4*>(trig + d / 2), sn = *reinterpret_cast<const f32x4*>(trig + rot / 2 + d / 2);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              const float u = bf16lo_to_f32(raw[e]), v = bf16hi_to_f32(raw[e]);
              w[e] = pack_bf16x2(u * cs[e] - v * sn[e], v * cs[e] + u * sn[e]);
            }
          } else {
#pragma unroll 1
            for (int e = 0; e < 8; ++e) {
              const int k = c + e;
              uint32_t bits = 0;
              if (k < kv_rank) {
                bits = ql[k];
              } else if (k < width) {
                const int d = k - kv_rank, i2 = d >> 1;
                const float u = bf16lo_to_f32(qr[2 * i2]), v = bf16lo_to_f32(qr[2 * i2 + 1]), cs = trig[i2], sn = trig[rot / 2 + i2];
                bits = f32_to_bf16_bits((d & 1) ? v * cs + u * sn : u * cs - v * sn);
              }
              tile[hr * lp + k] = (uint16_t)bits;
            }
            continue;
          }
        }
        store16(tile + hr * lp + c, w);
      }
    }
    __syncthreads();
    bf16x8 qb[NQ];
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
      const int ks = 2 * i + kh;
      qb[i] = ks < ksteps ? tile_row(tile, lp, n, 32 * ks + 8 * jj) : __builtin_bit_cast(bf16x8, u32x4{0u, 0u, 0u, 0u});
    }

    f32x4 acc[NT];
#pragma unroll
    for (int i = 0; i < NT; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m_run = -INFINITY, l_run = 0.f;

    for (int tok0 = tok_begin; tok0 < tok_end; tok0 += kTileTokens) {
      const bool ok = ok_next;
      __syncthreads();      // the last tile (or the query rows) have been read
#pragma unroll
      for (int j = 0; j < NQ; ++j)
        if (pr[j] < kTileTokens) store16(tile + pr[j] * lp + pc[j], reg[j]);
      __syncthreads();
      if (tok0 + kTileTokens < tok_end) ok_next = issue(tok0 + kTileTokens);
      f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < NQ; ++i) {
        const int ks = 2 * i + kh;
        if (ks < ksteps) s = mfma16(tile_row(tile, lp, 16 * tt + n, 32 * ks + 8 * jj), qb[i], s);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) part_s[kh][16 * tt + 4 * jj + e][n] = s[e];
      __syncthreads();
      const int valid = ok ? tok_end - tok0 : 0;
      float sv[8], m_loc = -INFINITY;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int t = 4 * jj + (e & 3) + 16 * (e >> 2);
        sv[e] = t < valid ? (part_s[0][t][n] + part_s[1][t][n]) * scale_log2 : -INFINITY;
        m_loc = fmaxf(m_loc, sv[e]);
      }
      m_loc = fmaxf(m_loc, __shfl_xor(m_loc, 16, kWave));
      m_loc = fmaxf(m_loc, __shfl_xor(m_loc, 32, kWave));
      const float m_new = fmaxf(m_run, m_loc);
      const float m_safe = m_new == -INFINITY ? 0.f : m_new;
      const float alpha = __builtin_amdgcn_exp2f(m_run - m_safe);
      float pv[8], psum = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        pv[e] = __builtin_amdgcn_exp2f(sv[e] - m_safe);
        psum += pv[e];
      }
      l_run = l_run * alpha + psum;
      m_run = m_new;
      if (__any(alpha != 1.0f)) {
#pragma unroll
        for (int i = 0; i < NT; ++i) acc[i] *= alpha;
      }
      bf16x8 hi, lo;
      split8(pv, hi, lo);
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        const int c0 = 16 * (wave + 4 * i);
        if (c0 < kv_rank) {
          const bf16x8 ca = __builtin_bit_cast(bf16x8, join(tile_block_columns(tile, lp, 4 * jj, c0, lane), tile_block_columns(tile, lp, 16 + 4 * jj, c0, lane)));
          acc[i] = mfma16(ca, hi, acc[i]);
          acc[i] = mfma16(ca, lo, acc[i]);
        }
      }
    }
    float l_tot = l_run + __shfl_xor(l_run, 16, kWave);
    l_tot += __shfl_xor(l_tot, 32, kWave);
    if (h >= heads) continue;
    if (run == row_tiles) {
      const float inv = l_tot > 0.f ? 1.0f / l_tot : 0.f;
      uint16_t* orow = (uint16_t*)a.out + ((int64_t)row * heads + h) * kv_rank;
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        const int r = 16 * (wave + 4 * i) + 4 * jj;
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (r + e < kv_rank) orow[r + e] = (uint16_t)f32_to_bf16_bits(acc[i][e] * inv);
      }
      continue;
    }
    const int64_t slot = (((int64_t)ht * p.columns + column) * 2 + (tile0 > 0 ? 0 : 1)) * kHeadTile + n;
    float* prow = p.part + slot * kv_rank;
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int r = 16 * (wave + 4 * i) + 4 * jj;
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (r + e < kv_rank) prow[r + e] = acc[i][e];
    }
    if (wave == 0 && jj == 0) {
      p.ml[2 * slot] = m_run;
      p.ml[2 * slot + 1] = l_tot;
    }
  }
}

// One wave per (row, head).
__global__ __launch_bounds__(64) void latent_combine_kernel(const LatentDecodeArgs p) {
  const mops_hip_latent_rows& a = p.a;
  const int heads = (int)a.heads, kv_rank = (int)a.kv_rank;
  const int h = blockIdx.x % heads, row = blockIdx.x / heads, lane = threadIdx.x;
  const int per = p.plan[0], f0 = p.plan[1 + row], f1 = p.plan[2 + row];
  uint16_t* out = (uint16_t*)a.out + ((int64_t)row * heads + h) * kv_rank;
  if (f1 <= f0) {
    for (int r = lane; r < kv_rank; r += kWave) out[r] = 0;
    return;
  }
  const int j0 = f0 / per, j1 = (f1 - 1) / per;
  if (j0 == j1) return;
  // slot 1 in the run where the row begins, slot 0 in the following ones
  auto slot_of = [&](int j) {
    return (((int64_t)(h / kHeadTile) * p.columns + j) * 2 + (j == j0 ? 1 : 0)) * kHeadTile + h % kHeadTile;
  };
  float m = -INFINITY;
  for (int j = j0 + lane; j <= j1; j += kWave) m = fmaxf(m, p.ml[2 * slot_of(j)]);
  m = group_max<kWave>(m);
  const float safe = m == -INFINITY ? 0.f : m;
  float l = 0.f;
  for (int j = j0 + lane; j <= j1; j += kWave) l += __builtin_amdgcn_exp2f(p.ml[2 * slot_of(j)] - safe) * p.ml[2 * slot_of(j) + 1];
  l = group_sum<kWave>(l);
  const float inv = l > 0.f ? 1.0f / l : 0.f;
  for (int r0 = 0; r0 < kv_rank; r0 += 8 * kWave) {
    float o[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    for (int j = j0; j <= j1; ++j) {
      const int64_t s = slot_of(j);
      const float w = __builtin_amdgcn_exp2f(p.ml[2 * s] - safe);
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int r = r0 + e * kWave + lane;
        if (r < kv_rank) o[e] += w * p.part[s * kv_rank + r];
      }
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int r = r0 + e * kWave + lane;
      if (r < kv_rank) out[r] = (uint16_t)f32_to_bf16_bits(o[e] * inv);
    }
  }
}

int check_latent_rows(const mops_hip_latent_rows* a);   // latent_attention.hip

// Two workgroups per CU for wide latents, more where registers and LDS allow.
static int column_count(int64_t width, int64_t kv_rank, int64_t head_tiles) {
  const int wgs = width <= 128 && kv_rank <= 128 ? 1024 : (width <= 320 && kv_rank <= 256 ? 768 : 512);
  const int64_t c = wgs / head_tiles;
  return c < 32 ? 32 : (int)c;
}
static int64_t plan_bytes(int64_t rows) { return ((rows + 2) * 4 + 255) / 256 * 256; }

}  // namespace mops

extern "C" int64_t mops_hip_latent_decode_workspace_bytes(int64_t rows, int64_t heads, int64_t kv_rank, int64_t rot_dim) {
  using namespace mops;
  if (rows <= 0 || heads <= 0 || kv_rank <= 0 || rot_dim < 0) return 0;
  const int64_t ht = (heads + kHeadTile - 1) / kHeadTile;
  return plan_bytes(rows) + ht * column_count(kv_rank + rot_dim, kv_rank, ht) * 2 * kHeadTile * (kv_rank + 2) * (int64_t)sizeof(float);
}

extern "C" int mops_hip_latent_decode(const mops_hip_latent_rows* a, void* workspace, int64_t workspace_bytes, void* stream) {
  using namespace mops;
  const int pre = check_latent_rows(a);
  if (pre != 1) return pre;
  const int64_t width = a->kv_rank + a->rot_dim;
  if (a->dtype != MOPS_HIP_BF16 || width > 576 || a->kv_rank > 512 || a->block_size % kTileTokens || a->pitch % 8) return MOPS_HIP_EUNSUPPORTED;
  if (!aligned16(a->cache)) return MOPS_HIP_EALIGN;
  const int64_t tokens = a->max_blocks * a->block_size;
  if (tokens > 0x7fffffffLL - kTileTokens || a->rows * ((tokens + kTileTokens - 1) / kTileTokens) > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  LatentDecodeArgs p;
  p.a = *a;
  p.head_tiles = (int)((a->heads + kHeadTile - 1) / kHeadTile);
  p.columns = column_count(width, a->kv_rank, p.head_tiles);
  if (!workspace || workspace_bytes < mops_hip_latent_decode_workspace_bytes(a->rows, a->heads, a->kv_rank, a->rot_dim)) return MOPS_HIP_EWORKSPACE;
  if (!aligned16(workspace)) return MOPS_HIP_EALIGN;
  p.plan = (int*)workspace;
  p.part = (float*)((char*)workspace + plan_bytes(a->rows));
  p.ml = p.part + (int64_t)p.head_tiles * p.columns * 2 * kHeadTile * a->kv_rank;
  p.vec_q = a->kv_rank % 8 == 0 && a->rot_dim % 8 == 0 && a->q_rot_token_stride % 8 == 0 && a->q_rot_head_stride % 8 == 0 &&
            aligned16(a->q_latent) && aligned16(a->q_rot) && aligned16(a->cos_sin);
  const dim3 grid((unsigned)(p.columns * p.head_tiles));
  hipStream_t s = (hipStream_t)stream;
  if (width <= 128 && a->kv_rank <= 128) hipLaunchKernelGGL((latent_decode_kernel<2, 2>), grid, dim3(256), 0, s, p);
  else if (width <= 320 && a->kv_rank <= 256) hipLaunchKernelGGL((latent_decode_kernel<5, 4>), grid, dim3(256), 0, s, p);
  else hipLaunchKernelGGL((latent_decode_kernel<9, 8>), grid, dim3(256), 0, s, p);
  hipLaunchKernelGGL(latent_combine_kernel, dim3((unsigned)(a->rows * a->heads)), dim3(64), 0, s, p);
  return finish_launch();
}
