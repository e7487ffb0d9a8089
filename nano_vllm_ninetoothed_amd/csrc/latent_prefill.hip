// Latent attention for long portions (bf16): keys and values of the whole context are expanded once, then an ordinary causal
// attention with per-head keys [dim | shared rotated part] and values [vdim] runs on the matrix cores.
//
//   latent_gather          the latent rows and key parts of each sequence's context, out of the pages into packed rows whose
//                          per-sequence base is a multiple of 64 (rows behind the context are zeros)
//   (two library GEMMs)    K = c W_uk^T [rows, heads * dim],  V^T = W_uv c^T [heads * vdim, rows]
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

constexpr int kKeys = 64, kKeyPitch = kKeys + 8;      // queries per workgroup: 4 waves x 32

struct LatentPrefillArgs {
  const uint16_t* q;              // [tokens][heads][dim + rot], rotated part raw
  int64_t q_token_stride, q_head_stride;
  const uint16_t *k, *kr, *vt;
  int64_t k_stride, kr_stride, vt_stride;
  const int32_t* tiles;           // [n][5]: first query token, queries, position of the first, first key row, keys
  int num_tiles;
  uint16_t* out;                  // [tokens][heads][vdim]
  const float* cos_sin;
  int64_t max_positions;
  int heads, dim, rot, vdim;
  float scale_log2;
  bool vec_q, vec_k, vec_out;
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
  const int nk = (dk + 15) >> 4, nv = (a.vdim + 31) >> 5;
  const int qi = 32 * wave + col;                       // this lane's query of the tile
  const bool q_ok = qi < q_count;
  const int pos = pos0 + qi;

  bf16x8 qb[NK];
  {
    const uint16_t* qr = a.q + (int64_t)(q_begin + (q_ok ? qi : 0)) * a.q_token_stride + h * a.q_head_stride;
    const float* trig = a.cos_sin + (int64_t)(pos < a.max_positions ? pos : a.max_positions - 1) * a.rot;
#pragma unroll
    for (int kk = 0; kk < NK; ++kk) {
      const int c = 16 * kk + 8 * hh;
      u32x4 w = {0u, 0u, 0u, 0u};
      if (q_ok && c < dk) {
        if (a.vec_q && c + 8 <= a.dim) {
          w = load16(qr + c);
        } else {
#pragma unroll
          for (int e = 0; e < 8; ++e) {
            const int i = c + e;
            uint32_t bits = 0;
            if (i < a.dim) {
              bits = qr[i];
            } else if (i < dk) {
              const int d = i - a.dim, i2 = d >> 1;
              const float u = bf16lo_to_f32(qr[a.dim + 2 * i2]), v = bf16lo_to_f32(qr[a.dim + 2 * i2 + 1]);
              const float cs = trig[i2], sn = trig[a.rot / 2 + i2];
              bits = f32_to_bf16_bits((d & 1) ? v * cs + u * sn : u * cs - v * sn);
            }
            w[e >> 1] |= bits << (16 * (e & 1));
          }
        }
      }
      qb[kk] = __builtin_bit_cast(bf16x8, w);
    }
  }

  f32x16 o[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[i][r] = 0.f;
  float m_run = -INFINITY, l_run = 0.f;

  const int visible = pos0 + q_count < keys ? pos0 + q_count : keys;      // keys any query of the tile sees
  const uint16_t* kbase = a.k + (int64_t)key_row0 * a.k_stride + (int64_t)h * a.dim;
  const uint16_t* krbase = a.kr + (int64_t)key_row0 * a.kr_stride;
  const uint16_t* vbase = a.vt + (int64_t)h * a.vdim * a.vt_stride + key_row0;
  u32x4 kreg[kKPieces > 0 ? kKPieces : 1], vreg[kVPieces];
  auto issue = [&](int k0) {
#pragma unroll
    for (int j = 0; j < kKPieces; ++j) {
      const int i = tid + 256 * j, r = i / (NK * 2), c = (i % (NK * 2)) * 8;
      u32x4 w = {0u, 0u, 0u, 0u};
      if (c < dk) {
        const uint16_t* kr = kbase + (int64_t)(k0 + r) * a.k_stride;
        const uint16_t* rr = krbase + (int64_t)(k0 + r) * a.kr_stride;
        if (a.vec_k) {
          w = c < a.dim ? load16(kr + c) : load16(rr + (c - a.dim));
        } else {
#pragma unroll
          for (int e = 0; e < 8; ++e) {
            const int d = c + e;
            const uint32_t bits = d < a.dim ? kr[d] : (d < dk ? rr[d - a.dim] : 0u);
            w[e >> 1] |= bits << (16 * (e & 1));
          }
        }
      }
      kreg[j] = w;
    }
#pragma unroll
    for (int j = 0; j < kVPieces; ++j) {
      const int i = tid + 256 * j, r = i / (kKeys / 8), c = (i % (kKeys / 8)) * 8;
      vreg[j] = r < a.vdim ? load16(vbase + (int64_t)r * a.vt_stride + k0 + c) : u32x4{0u, 0u, 0u, 0u};
    }
  };
  issue(0);
  for (int k0 = 0; k0 < visible; k0 += kKeys) {
    __syncthreads();
#pragma unroll
    for (int j = 0; j < kKPieces; ++j) {
      const int i = tid + 256 * j;
      store16(tk + (i / (NK * 2)) * kPitch + (i % (NK * 2)) * 8, kreg[j]);
    }
#pragma unroll
    for (int j = 0; j < kVPieces; ++j) {
      const int i = tid + 256 * j;
      store16(tv + (i / (kKeys / 8)) * kKeyPitch + (i % (kKeys / 8)) * 8, vreg[j]);
    }
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
      if (kk < nk) {
#pragma unroll
        for (int kt = 0; kt < 2; ++kt) s[kt] = mfma32(tile_row(tk, kPitch, 32 * kt + col, 16 * kk + 8 * hh), qb[kk], s[kt]);
      }
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
      for (int i = 0; i < NV; ++i)
        if (i < nv) o[i] *= alpha;
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
        // the keys of these eight values: j0 .. j0+3 and j0+8 .. j0+11
        const int j0 = 32 * kt + 16 * ks + 4 * hh;
#pragma unroll
        for (int i = 0; i < NV; ++i)
          if (i < nv) {
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

extern "C" int mops_hip_latent_prefill(const void* q, int64_t q_token_stride, int64_t q_head_stride, const void* k, int64_t k_stride,
                                       const void* kr, int64_t kr_stride, const void* vt, int64_t vt_stride, const int32_t* tiles,
                                       int64_t num_tiles, void* out, const float* cos_sin, int64_t max_positions, int64_t heads, int64_t dim,
                                       int64_t rot_dim, int64_t vdim, float scale, void* stream) {
  using namespace mops;
  if (num_tiles < 0 || heads <= 0 || dim <= 0 || rot_dim < 0 || (rot_dim & 1) || vdim <= 0 || max_positions <= 0) return MOPS_HIP_EINVAL;
  if (num_tiles == 0) return MOPS_HIP_OK;
  if (!q || !k || !kr || !vt || !tiles || !out || !cos_sin) return MOPS_HIP_EINVAL;
  if (q_head_stride < dim + rot_dim || k_stride < heads * dim || kr_stride < rot_dim) return MOPS_HIP_EINVAL;
  if (dim + rot_dim > 256 || vdim > 256 || heads > 65535 || num_tiles * heads > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  if (vt_stride % 8 || !aligned16(vt)) return MOPS_HIP_EALIGN;
  LatentPrefillArgs a;
  a.q = (const uint16_t*)q; a.q_token_stride = q_token_stride; a.q_head_stride = q_head_stride;
  a.k = (const uint16_t*)k; a.kr = (const uint16_t*)kr; a.vt = (const uint16_t*)vt;
  a.k_stride = k_stride; a.kr_stride = kr_stride; a.vt_stride = vt_stride;
  a.tiles = tiles; a.num_tiles = (int)num_tiles; a.out = (uint16_t*)out; a.cos_sin = cos_sin; a.max_positions = max_positions;
  a.heads = (int)heads; a.dim = (int)dim; a.rot = (int)rot_dim; a.vdim = (int)vdim;
  a.scale_log2 = scale * 1.4426950408889634f;
  a.vec_q = dim % 8 == 0 && q_token_stride % 8 == 0 && q_head_stride % 8 == 0 && aligned16(q);
  a.vec_k = dim % 8 == 0 && rot_dim % 8 == 0 && k_stride % 8 == 0 && kr_stride % 8 == 0 && aligned16(k) && aligned16(kr);
  a.vec_out = vdim % 4 == 0 && aligned16(out);
  const dim3 grid((unsigned)(num_tiles * heads)), block(256);
  hipStream_t s = (hipStream_t)stream;
  const int64_t dk = dim + rot_dim;
#define MOPS_LP(K, V) hipLaunchKernelGGL((latent_prefill_kernel<K, V>), grid, block, 0, s, a)
  if (vdim <= 128) {
    if (dk <= 64) MOPS_LP(4, 4);
    else if (dk <= 128) MOPS_LP(8, 4);
    else if (dk <= 192) MOPS_LP(12, 4);
    else MOPS_LP(16, 4);
  } else {
    MOPS_LP(16, 8);
  }
#undef MOPS_LP
  return finish_launch();
}
