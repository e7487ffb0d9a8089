// Latent attention for long portions (bf16): keys and values of the whole context are expanded once, then an ordinary causal
// attention with per-head keys [dim | shared rotated part] and values [vdim] runs on the matrix cores.
//
//   latent_gather          the latent rows and key parts of each sequence's context, out of the pages into packed rows whose
//                          per-sequence base is a multiple of 64 (rows behind the context are zeros)
//   (two library GEMMs)    K = c W_uk^T [rows, heads * dim],  V^T = W_uv c^T [heads * vdim, rows]
//   rotate_pairs           the rotated part of the queries, in place
//   latent_prefill_kernel  workgroup (four waves) = (128 query tokens, head); a wave takes 32 queries.  64-key tiles of K and
//                          V^T in LDS, the next tile in flight into registers.  v_mfma_f32_32x32x16_bf16 throughout:
//       S^T [key, query] = K Q^T        the softmax runs over keys: in a lane and its partner in the other half
//       O^T [v, query]  += V^T P^T      P from the accumulators of S^T (same lane), as the sum of two bf16 numbers
#include "mfma_tiles.h"

namespace mops {

__global__ __launch_bounds__(256) void latent_gather_kernel(const uint16_t* __restrict__ cache, int pitch, const int32_t* __restrict__ block_table,
                                                            int64_t table_stride, int block_size, int64_t num_blocks, int64_t max_blocks,
                                                            const int32_t* __restrict__ row_seq, const int32_t* __restrict__ row_pos,
                                                            uint16_t* __restrict__ c, int c_pitch, uint16_t* __restrict__ kr, int kr_pitch,
                                                            int64_t rows, int kv_rank, int rot) {
  const int64_t row = (int64_t)blockIdx.x * 4 + threadIdx.x / kWave;
  if (row >= rows) return;
  const int lane = threadIdx.x & (kWave - 1);
  const int pos = row_pos[row];
  const uint16_t* src = nullptr;
  if (pos >= 0 && pos / block_size < max_blocks) {
    const int id = block_table[(int64_t)row_seq[row] * table_stride + pos / block_size];
    if (id >= 0 && id < num_blocks) src = cache + ((int64_t)id * block_size + pos % block_size) * pitch;
  }
  uint16_t* cr = c + row * c_pitch;
  if (kv_rank % 8 == 0) {
    for (int i = lane * 8; i < kv_rank; i += kWave * 8) store16(cr + i, src ? load16(src + i) : u32x4{0u, 0u, 0u, 0u});
    for (int i = kv_rank + lane; i < c_pitch; i += kWave) cr[i] = 0;
  } else {
    for (int i = lane; i < c_pitch; i += kWave) cr[i] = src && i < kv_rank ? src[i] : (uint16_t)0;
  }
  for (int i = lane; i < kr_pitch; i += kWave) kr[row * kr_pitch + i] = src && i < rot ? src[kv_rank + i] : (uint16_t)0;
}

// One 16-byte piece (four pairs) or one pair per thread, in place.
template <int PAIRS>
__global__ __launch_bounds__(256) void rotate_pairs_kernel(uint16_t* __restrict__ x, int64_t token_stride, int64_t head_stride,
                                                           const int32_t* __restrict__ positions, const float* __restrict__ cos_sin,
                                                           int64_t max_positions, int64_t tokens, int heads, int rot) {
  const int per_head = rot / (2 * PAIRS);
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= tokens * heads * per_head) return;
  const int j = (int)(i % per_head) * PAIRS;
  const int h = (int)(i / per_head % heads);
  const int64_t t = i / per_head / heads;
  const int64_t pos = positions[t] < max_positions ? positions[t] : max_positions - 1;
  const float* trig = cos_sin + pos * rot + j;
  bf16_t* p = reinterpret_cast<bf16_t*>(x + t * token_stride + h * head_stride + 2 * j);
  float v[2 * PAIRS];
  load_vec<2 * PAIRS>(p, v);
#pragma unroll
  for (int e = 0; e < PAIRS; ++e) {
    const float c = trig[e], s = trig[rot / 2 + e], a = v[2 * e], b = v[2 * e + 1];
    v[2 * e] = a * c - b * s;
    v[2 * e + 1] = b * c + a * s;
  }
  store_vec<2 * PAIRS>(p, v);
}

constexpr int kKeys = 64, kKeyPitch = kKeys + 8;      // queries per workgroup: 4 waves x 32

struct LatentPrefillArgs {
  const uint16_t* q;              // [tokens][heads][dim + rot]
  int64_t q_token_stride, q_head_stride;
  const uint16_t *k, *kr, *vt;
  int64_t k_stride, kr_stride, vt_stride;
  const int32_t* tiles;           // [n][5]: first query token, queries, position of the first, first key row, keys
  int num_tiles;
  uint16_t* out;                  // [tokens][heads][vdim]
  int heads, dim, rot, vdim;
  float scale_log2;
  bool vec_out;
};

// NK: 16-wide k steps (dim + rot <= 16 NK), NV: 32-wide pieces of the value (vdim <= 32 NV)
template <int NK, int NV>
__global__ __launch_bounds__(256, 2) void latent_prefill_kernel(const LatentPrefillArgs a) {
  constexpr int kPitch = NK * 16 + 8;
  constexpr int kKPieces = kKeys * NK * 2 / 256;       // 16-byte pieces of K per thread
  constexpr int kVPieces = NV * 32 * (kKeys / 8) / 256;
  __shared__ __align__(16) uint16_t tk[kKeys * kPitch];
  __shared__ __align__(16) uint16_t tv[NV * 32 * kKeyPitch];
  const int h = blockIdx.x % a.heads;
  const int32_t* t = a.tiles + 5 * (int64_t)(blockIdx.x / a.heads);
  const int q_begin = t[0], q_count = t[1], pos0 = t[2], key_row0 = t[3], keys = t[4];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 31, hh = lane >> 5;
  const int dk = a.dim + a.rot;
  const int qi = 32 * wave + col;                       // this lane's query of the tile
  const bool q_ok = qi < q_count;
  const int pos = pos0 + qi;

  bf16x8 qb[NK];
  {
    const uint16_t* qr = a.q + (int64_t)(q_begin + (q_ok ? qi : 0)) * a.q_token_stride + h * a.q_head_stride;
#pragma unroll
    for (int kk = 0; kk < NK; ++kk) {
      const int c = 16 * kk + 8 * hh;
      qb[kk] = __builtin_bit_cast(bf16x8, q_ok && c < dk ? load16(qr + c) : u32x4{0u, 0u, 0u, 0u});
    }
  }

  f32x16 o[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[i][r] = 0.f;
  float m_run = -INFINITY, l_run = 0.f;

  const int visible = pos0 + q_count < keys ? pos0 + q_count : keys;      // keys any query of the tile sees
  // thread -> pieces of 16 bytes: a key row belongs to four threads, a row of V^T to eight
  const int krow = tid >> 2, kcol = (tid & 3) * 8, vrow = tid >> 3, vcol = (tid & 7) * 8;
  const uint16_t* kp = a.k + (int64_t)(key_row0 + krow) * a.k_stride + (int64_t)h * a.dim;
  const uint16_t* krp = a.kr + (int64_t)(key_row0 + krow) * a.kr_stride - a.dim;
  const uint16_t* vp = a.vt + ((int64_t)h * a.vdim + vrow) * a.vt_stride + key_row0 + vcol;
  u32x4 kreg[kKPieces], vreg[kVPieces];
  auto issue = [&](int k0) {
#pragma unroll
    for (int j = 0; j < kKPieces; ++j) {
      const int c = kcol + 32 * j;
      const uint16_t* src = c < a.dim ? kp + (int64_t)k0 * a.k_stride : krp + (int64_t)k0 * a.kr_stride;
      kreg[j] = c < dk ? load16(src + c) : u32x4{0u, 0u, 0u, 0u};
    }
#pragma unroll
    for (int j = 0; j < kVPieces; ++j)
      vreg[j] = vrow + 32 * j < a.vdim ? load16(vp + (int64_t)(32 * j) * a.vt_stride + k0) : u32x4{0u, 0u, 0u, 0u};
  };
  issue(0);
  for (int k0 = 0; k0 < visible; k0 += kKeys) {
    __syncthreads();
#pragma unroll
    for (int j = 0; j < kKPieces; ++j) store16(tk + krow * kPitch + kcol + 32 * j, kreg[j]);
#pragma unroll
    for (int j = 0; j < kVPieces; ++j) store16(tv + (vrow + 32 * j) * kKeyPitch + vcol, vreg[j]);
    __syncthreads();
    if (k0 + kKeys < visible) issue(k0 + kKeys);
    if (k0 > pos0 + 32 * wave + 31) continue;           // this wave's queries see none of the tile
    f32x16 s[2];
#pragma unroll
    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
      for (int r = 0; r < 16; ++r) s[kt][r] = 0.f;
#pragma unroll
    for (int kk = 0; kk < NK; ++kk)
#pragma unroll
      for (int kt = 0; kt < 2; ++kt) s[kt] = mfma32(tile_row(tk, kPitch, 32 * kt + col, 16 * kk + 8 * hh), qb[kk], s[kt]);
    float m_loc = -INFINITY;
    const int last = pos < keys - 1 ? pos : keys - 1;
    if (k0 + kKeys - 1 > pos0 + 32 * wave || k0 + kKeys > keys) {      // the diagonal or the end of the context: mask
#pragma unroll
      for (int kt = 0; kt < 2; ++kt)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int key = k0 + 32 * kt + 8 * (r >> 2) + 4 * hh + (r & 3);
          s[kt][r] = key <= last ? s[kt][r] * a.scale_log2 : -INFINITY;
          m_loc = fmaxf(m_loc, s[kt][r]);
        }
    } else {
#pragma unroll
      for (int kt = 0; kt < 2; ++kt)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          s[kt][r] *= a.scale_log2;
          m_loc = fmaxf(m_loc, s[kt][r]);
        }
    }
    m_loc = fmaxf(m_loc, __shfl_xor(m_loc, 32, kWave));
    const float m_new = fmaxf(m_run, m_loc);
    const float m_safe = m_new == -INFINITY ? 0.f : m_new;
    const float alpha = __builtin_amdgcn_exp2f(m_run - m_safe);
    m_run = m_new;
    if (__any(alpha != 1.0f)) {
      l_run *= alpha;
#pragma unroll
      for (int i = 0; i < NV; ++i) o[i] *= alpha;
    }
#pragma unroll
    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        float pv[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          pv[e] = __builtin_amdgcn_exp2f(s[kt][8 * ks + e] - m_safe);
          l_run += pv[e];
        }
        bf16x8 hi, lo;
        split8(pv, hi, lo);
        __builtin_amdgcn_sched_barrier(0);      // keeps the operand reads of the next step out of this one's registers
        // the keys of these eight values: j0 .. j0+3 and j0+8 .. j0+11
        const int j0 = 32 * kt + 16 * ks + 4 * hh;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
          const uint16_t* vr = tv + (32 * i + col) * kKeyPitch + j0;
          const u32x2 w0 = *reinterpret_cast<const u32x2*>(vr), w1 = *reinterpret_cast<const u32x2*>(vr + 8);
          const bf16x8 va = __builtin_bit_cast(bf16x8, u32x4{w0[0], w0[1], w1[0], w1[1]});
          o[i] = mfma32(va, hi, o[i]);
          o[i] = mfma32(va, lo, o[i]);
        }
      }
  }
  if (!q_ok) return;
  const float l = l_run + __shfl_xor(l_run, 32, kWave);
  const float inv = l > 0.f ? 1.0f / l : 0.f;
  uint16_t* orow = a.out + ((int64_t)(q_begin + qi) * a.heads + h) * a.vdim;
#pragma unroll
  for (int i = 0; i < NV; ++i)
#pragma unroll
    for (int q4 = 0; q4 < 4; ++q4) {
      const int v = 32 * i + 8 * q4 + 4 * hh;
      if (a.vec_out && v + 4 <= a.vdim) {
        *reinterpret_cast<u32x2*>(orow + v) = u32x2{pack_bf16x2(o[i][4 * q4] * inv, o[i][4 * q4 + 1] * inv),
                                                    pack_bf16x2(o[i][4 * q4 + 2] * inv, o[i][4 * q4 + 3] * inv)};
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (v + e < a.vdim) orow[v + e] = (uint16_t)f32_to_bf16_bits(o[i][4 * q4 + e] * inv);
      }
    }
}

}  // namespace mops

extern "C" int mops_hip_latent_gather(const void* cache, int64_t pitch, const int32_t* block_table, int64_t table_stride, int64_t block_size,
                                      int64_t num_blocks, int64_t max_blocks, const int32_t* row_seq, const int32_t* row_pos, void* c,
                                      int64_t c_pitch, void* kr, int64_t kr_pitch, int64_t rows, int64_t kv_rank, int64_t rot_dim, void* stream) {
  using namespace mops;
  if (rows < 0 || kv_rank <= 0 || rot_dim < 0 || pitch < kv_rank + rot_dim || c_pitch < kv_rank || kr_pitch < rot_dim || block_size <= 0 ||
      num_blocks <= 0 || max_blocks <= 0 || table_stride < max_blocks)
    return MOPS_HIP_EINVAL;
  if (rows == 0) return MOPS_HIP_OK;
  if (!cache || !block_table || !row_seq || !row_pos || !c || !kr) return MOPS_HIP_EINVAL;
  if (!aligned16(cache) || pitch % 8 || !aligned16(c) || c_pitch % 8) return MOPS_HIP_EALIGN;
  if (rows > (1 << 28) || c_pitch > (1 << 20) || kr_pitch > (1 << 20) || block_size > (1 << 20)) return MOPS_HIP_EUNSUPPORTED;
  hipLaunchKernelGGL(latent_gather_kernel, dim3((unsigned)((rows + 3) / 4)), dim3(256), 0, (hipStream_t)stream, (const uint16_t*)cache, (int)pitch,
                     block_table, table_stride, (int)block_size, num_blocks, max_blocks, row_seq, row_pos, (uint16_t*)c, (int)c_pitch, (uint16_t*)kr,
                     (int)kr_pitch, rows, (int)kv_rank, (int)rot_dim);
  return finish_launch();
}

extern "C" int mops_hip_rotate_pairs(void* x, int64_t token_stride, int64_t head_stride, const int32_t* positions, const float* cos_sin,
                                     int64_t max_positions, int64_t tokens, int64_t heads, int64_t rot, void* stream) {
  using namespace mops;
  if (tokens < 0 || heads <= 0 || rot < 0 || (rot & 1) || max_positions <= 0) return MOPS_HIP_EINVAL;
  if (tokens == 0 || rot == 0) return MOPS_HIP_OK;
  if (!x || !positions || !cos_sin || head_stride < rot) return MOPS_HIP_EINVAL;
  const bool vec = rot % 8 == 0 && token_stride % 8 == 0 && head_stride % 8 == 0 && aligned16(x);
  const int64_t wgs = (tokens * heads * (rot / (vec ? 8 : 2)) + 255) / 256;
  if (wgs > 0x7fffffffLL || heads > 65536 || rot > 65536) return MOPS_HIP_EUNSUPPORTED;
  if (vec)
    hipLaunchKernelGGL((rotate_pairs_kernel<4>), dim3((unsigned)wgs), dim3(256), 0, (hipStream_t)stream, (uint16_t*)x, token_stride, head_stride,
                       positions, cos_sin, max_positions, tokens, (int)heads, (int)rot);
  else
    hipLaunchKernelGGL((rotate_pairs_kernel<1>), dim3((unsigned)wgs), dim3(256), 0, (hipStream_t)stream, (uint16_t*)x, token_stride, head_stride,
                       positions, cos_sin, max_positions, tokens, (int)heads, (int)rot);
  return finish_launch();
}

extern "C" int mops_hip_latent_prefill(const void* q, int64_t q_token_stride, int64_t q_head_stride, const void* k, int64_t k_stride,
                                       const void* kr, int64_t kr_stride, const void* vt, int64_t vt_stride, const int32_t* tiles,
                                       int64_t num_tiles, void* out, int64_t heads, int64_t dim, int64_t rot_dim, int64_t vdim, float scale,
                                       void* stream) {
  using namespace mops;
  if (num_tiles < 0 || heads <= 0 || dim <= 0 || rot_dim < 0 || vdim <= 0) return MOPS_HIP_EINVAL;
  if (num_tiles == 0) return MOPS_HIP_OK;
  if (!q || !k || !kr || !vt || !tiles || !out) return MOPS_HIP_EINVAL;
  if (q_head_stride < dim + rot_dim || k_stride < heads * dim || kr_stride < rot_dim) return MOPS_HIP_EINVAL;
  if (dim + rot_dim > 256 || vdim > 256 || heads > 65535 || num_tiles * heads > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  if (dim % 8 || rot_dim % 8 || q_token_stride % 8 || q_head_stride % 8 || k_stride % 8 || kr_stride % 8 || vt_stride % 8 || !aligned16(q) ||
      !aligned16(k) || !aligned16(kr) || !aligned16(vt))
    return MOPS_HIP_EALIGN;
  LatentPrefillArgs a;
  a.q = (const uint16_t*)q; a.q_token_stride = q_token_stride; a.q_head_stride = q_head_stride;
  a.k = (const uint16_t*)k; a.kr = (const uint16_t*)kr; a.vt = (const uint16_t*)vt;
  a.k_stride = k_stride; a.kr_stride = kr_stride; a.vt_stride = vt_stride;
  a.tiles = tiles; a.num_tiles = (int)num_tiles; a.out = (uint16_t*)out;
  a.heads = (int)heads; a.dim = (int)dim; a.rot = (int)rot_dim; a.vdim = (int)vdim;
  a.scale_log2 = scale * 1.4426950408889634f;
  a.vec_out = vdim % 4 == 0 && aligned16(out);
  const dim3 grid((unsigned)(num_tiles * heads)), block(256);
  hipStream_t s = (hipStream_t)stream;
  const int64_t dk = dim + rot_dim;
#define MOPS_LP(K, V) hipLaunchKernelGGL((latent_prefill_kernel<K, V>), grid, block, 0, s, a)
#define MOPS_LP_DK(V) do { if (dk <= 64) MOPS_LP(4, V); else if (dk <= 128) MOPS_LP(8, V); else if (dk <= 192) MOPS_LP(12, V); \
                           else MOPS_LP(16, V); } while (0)
  if (vdim <= 64) MOPS_LP_DK(2);
  else if (vdim <= 128) MOPS_LP_DK(4);
  else MOPS_LP(16, 8);
#undef MOPS_LP_DK
#undef MOPS_LP
  return finish_launch();
}
