// Query rows against the paged latent cache on the matrix cores (bf16): the form of latent_attention_rows for decode steps
// and short portions.  The cache row is key and value at once, so it is read once per 16 heads.
//
// Workgroup (four waves) = (row, 16 heads, run of `split` tokens), walking 32-token tiles: the next tile is in flight into
// registers while this one is used out of LDS.
//   S^T [token, head] = C Q^T    a wave takes 16 tokens and every second 32-wide k step; the two partial sums meet in LDS
//   softmax over tokens          every wave, redundantly, in the layout the next product reads
//   O^T [r, head] += C^T P^T     a wave takes every fourth 16-wide piece of the latent; C^T through transposing LDS reads,
//                                P as the sum of two bf16 numbers
// Rows whose context spans several runs leave (max, sum, unnormalised O) per run; latent_combine_kernel merges them.
#include "mfma_tiles.h"

namespace mops {

constexpr int kTileTokens = 32;
constexpr int kHeadTile = 16;

struct LatentDecodeArgs {
  mops_hip_latent_rows a;
  int split, max_splits, head_tiles;
  float* part;      // [rows][head_tiles][max_splits][16][kv_rank]
  float* ml;        // [rows][head_tiles][max_splits][16][2]
  bool vec_q;
};

// NQ: 32-wide k steps per wave (kv_rank + rot_dim <= 64 NQ); NT: 16-wide latent pieces per wave (kv_rank <= 64 NT)
template <int NQ, int NT>
__global__ __launch_bounds__(256, 2) void latent_decode_kernel(const LatentDecodeArgs p) {
  constexpr int kMaxPitch = 64 * NQ + 8;
  __shared__ __align__(16) uint16_t tile[kTileTokens * kMaxPitch];
  __shared__ __align__(16) float part_s[2][kTileTokens][kHeadTile + 1];
  const mops_hip_latent_rows& a = p.a;
  const int split_id = blockIdx.x % p.max_splits;
  const int ht = (blockIdx.x / p.max_splits) % p.head_tiles;
  const int64_t row = blockIdx.x / (p.max_splits * p.head_tiles);
  const int len = a.context_lens[row];
  const int tok_begin = split_id * p.split;
  const int heads = (int)a.heads, kv_rank = (int)a.kv_rank, rot = (int)a.rot_dim, width = kv_rank + rot;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int n = lane & 15, jj = lane >> 4;
  const int h = ht * kHeadTile + n;
  if (tok_begin >= len) {
    if (len <= 0 && split_id == 0)      // an empty context attends to nothing
      for (int i = tid; i < kHeadTile * kv_rank; i += 256) {
        const int hr = ht * kHeadTile + i / kv_rank;
        if (hr < heads) ((uint16_t*)a.out)[(row * heads + hr) * kv_rank + i % kv_rank] = 0;
      }
    return;
  }
  const int tok_end = len < tok_begin + p.split ? len : tok_begin + p.split;
  const int ksteps = (width + 31) >> 5, lp = ksteps * 32 + 8, row_pieces = ksteps * 4;
  const int seq = a.row_seq ? a.row_seq[row] : (int)row;
  const int32_t* table = a.block_table + (int64_t)seq * a.block_table_stride;
  const int bs = (int)a.block_size;

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
  bool ok_next = issue(tok_begin);

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
        const uint16_t* ql = (const uint16_t*)a.q_latent + (row * heads + head) * kv_rank;
        if (p.vec_q && c + 8 <= kv_rank) {
          w = load16(ql + c);
        } else {
          const uint16_t* qr = (const uint16_t*)a.q_rot + row * a.q_rot_token_stride + head * a.q_rot_head_stride;
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
  const int tt = wave & 1, kh = wave >> 1;
#pragma unroll
  for (int i = 0; i < NQ; ++i) {
    const int ks = 2 * i + kh;
    qb[i] = ks < ksteps ? tile_row(tile, lp, n, 32 * ks + 8 * jj) : __builtin_bit_cast(bf16x8, u32x4{0u, 0u, 0u, 0u});
  }

  f32x4 acc[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m_run = -INFINITY, l_run = 0.f;
  const float scale_log2 = a.scale * 1.4426950408889634f;

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
  if (h >= heads) return;
  if (len <= p.split) {
    const float inv = l_tot > 0.f ? 1.0f / l_tot : 0.f;
    uint16_t* orow = (uint16_t*)a.out + (row * heads + h) * kv_rank;
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int r = 16 * (wave + 4 * i) + 4 * jj;
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (r + e < kv_rank) orow[r + e] = (uint16_t)f32_to_bf16_bits(acc[i][e] * inv);
    }
    return;
  }
  const int64_t slot = ((row * p.head_tiles + ht) * p.max_splits + split_id) * kHeadTile + n;
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

// One wave per (row, head) with more than one run.
__global__ __launch_bounds__(64) void latent_combine_kernel(const LatentDecodeArgs p) {
  const mops_hip_latent_rows& a = p.a;
  const int heads = (int)a.heads, kv_rank = (int)a.kv_rank;
  const int h = blockIdx.x % heads;
  const int64_t row = blockIdx.x / heads;
  const int len = a.context_lens[row];
  if (len <= p.split) return;
  int runs = (len + p.split - 1) / p.split;
  if (runs > p.max_splits) runs = p.max_splits;
  const int64_t slot0 = ((row * p.head_tiles + h / kHeadTile) * p.max_splits) * kHeadTile + h % kHeadTile;
  const int lane = threadIdx.x;
  float m = -INFINITY;
  for (int i = lane; i < runs; i += kWave) m = fmaxf(m, p.ml[2 * (slot0 + (int64_t)i * kHeadTile)]);
  m = group_max<kWave>(m);
  const float safe = m == -INFINITY ? 0.f : m;
  float l = 0.f;
  for (int i = lane; i < runs; i += kWave) {
    const float* x = p.ml + 2 * (slot0 + (int64_t)i * kHeadTile);
    l += __builtin_amdgcn_exp2f(x[0] - safe) * x[1];
  }
  l = group_sum<kWave>(l);
  const float inv = l > 0.f ? 1.0f / l : 0.f;
  uint16_t* out = (uint16_t*)a.out + (row * heads + h) * kv_rank;
  for (int r0 = 0; r0 < kv_rank; r0 += 4 * kWave) {
    float o[4] = {0.f, 0.f, 0.f, 0.f};
    for (int i = 0; i < runs; ++i) {
      const int64_t s = slot0 + (int64_t)i * kHeadTile;
      const float w = __builtin_amdgcn_exp2f(p.ml[2 * s] - safe);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int r = r0 + e * kWave + lane;
        if (r < kv_rank) o[e] += w * p.part[s * kv_rank + r];
      }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int r = r0 + e * kWave + lane;
      if (r < kv_rank) out[r] = (uint16_t)f32_to_bf16_bits(o[e] * inv);
    }
  }
}

int check_latent_rows(const mops_hip_latent_rows* a);   // latent_attention.hip

static int run_tokens(int64_t rows, int64_t head_tiles, int64_t max_tokens) {
  // long runs cost less merging, short ones fill the chip: as long as leaves about four workgroups per CU
  int split = 1024;
  while (split > 64 && rows * head_tiles * ((max_tokens + split - 1) / split) < 1024) split >>= 1;
  return split;
}

}  // namespace mops

extern "C" int64_t mops_hip_latent_decode_workspace_bytes(int64_t rows, int64_t heads, int64_t kv_rank, int64_t max_blocks, int64_t block_size) {
  using namespace mops;
  if (rows <= 0 || heads <= 0 || kv_rank <= 0 || max_blocks <= 0 || block_size <= 0) return 0;
  const int64_t ht = (heads + kHeadTile - 1) / kHeadTile, tokens = max_blocks * block_size;
  const int64_t split = run_tokens(rows, ht, tokens);
  return rows * ht * ((tokens + split - 1) / split) * kHeadTile * (kv_rank + 2) * (int64_t)sizeof(float);
}

extern "C" int mops_hip_latent_decode(const mops_hip_latent_rows* a, void* workspace, int64_t workspace_bytes, void* stream) {
  using namespace mops;
  const int pre = check_latent_rows(a);
  if (pre != 1) return pre;
  const int64_t width = a->kv_rank + a->rot_dim;
  if (a->dtype != MOPS_HIP_BF16 || width > 576 || a->kv_rank > 512 || a->block_size % kTileTokens || a->pitch % 8) return MOPS_HIP_EUNSUPPORTED;
  if (!aligned16(a->cache)) return MOPS_HIP_EALIGN;
  LatentDecodeArgs p;
  p.a = *a;
  p.head_tiles = (int)((a->heads + kHeadTile - 1) / kHeadTile);
  const int64_t tokens = a->max_blocks * a->block_size;
  if (tokens > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  p.split = run_tokens(a->rows, p.head_tiles, tokens);
  p.max_splits = (int)((tokens + p.split - 1) / p.split);
  const int64_t need = mops_hip_latent_decode_workspace_bytes(a->rows, a->heads, a->kv_rank, a->max_blocks, a->block_size);
  if (!workspace || workspace_bytes < need) return MOPS_HIP_EWORKSPACE;
  if (!aligned16(workspace)) return MOPS_HIP_EALIGN;
  const int64_t slots = a->rows * p.head_tiles * p.max_splits * kHeadTile;
  if (slots / kHeadTile > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  p.part = (float*)workspace;
  p.ml = p.part + slots * a->kv_rank;
  p.vec_q = a->kv_rank % 8 == 0 && aligned16(a->q_latent);
  const dim3 grid((unsigned)(a->rows * p.head_tiles * p.max_splits));
  hipStream_t s = (hipStream_t)stream;
  if (width <= 128 && a->kv_rank <= 128) hipLaunchKernelGGL((latent_decode_kernel<2, 2>), grid, dim3(256), 0, s, p);
  else if (width <= 320 && a->kv_rank <= 256) hipLaunchKernelGGL((latent_decode_kernel<5, 4>), grid, dim3(256), 0, s, p);
  else hipLaunchKernelGGL((latent_decode_kernel<9, 8>), grid, dim3(256), 0, s, p);
  if (p.max_splits > 1) hipLaunchKernelGGL(latent_combine_kernel, dim3((unsigned)(a->rows * a->heads)), dim3(64), 0, s, p);
  return finish_launch();
}
