// rotary_prepare: what stands between the packed projections [q | k | v] of every token and attention over paged keys and values:
// an optional RMS norm per head on q and k (one weight for all heads), a rotation of their first `rot` elements by the token's
// position, q to its own rows, k and v to their pages.  Pair i of a rotation is (element i, element i + rot / 2), or with `neighbours`
// (element 2i, element 2i + 1).  A bias over [q | k | v] is added first.
//
// LANES lanes own one head of one token, eight elements each, and take the other half of a pair from the lane that holds it.  Heads
// wider than that, or of odd sizes: a wave per head, element by element, with the other half read again.
#include "mixed_types.h"

namespace mops {

template <typename T, int VEC, int LANES>
__global__ __launch_bounds__(256) void rotary_prepare_kernel(const mops_hip_rotary_prepare_args a, int items) {
  const int64_t item = (int64_t)blockIdx.x * (256 / LANES) + threadIdx.x / LANES;
  if (item >= a.tokens * items) return;      // whole groups of lanes leave; the sums below stay inside a group
  const int64_t t = item / items;
  int h = (int)(item % items);
  const int lane = threadIdx.x & (LANES - 1), heads = (int)a.heads, groups = (int)a.kv_heads, dim = (int)a.dim, vdim = (int)a.vdim;
  const int dp = (dim + 7) / 8 * 8, vp = (vdim + 7) / 8 * 8;
  const T* row = (const T*)a.qkv + t * a.qkv_stride;
  const int64_t slot = a.slot_mapping[t];
  const bool filed = slot >= 0 && slot < a.num_slots;
  if (h >= heads + groups) {      // a value head: copied
    h -= heads + groups;
    if (!filed) return;
    const T* src = row + (heads + groups) * dim + h * vdim;
    const T* bias = a.bias ? (const T*)a.bias + (heads + groups) * dim + h * vdim : nullptr;
    T* dst = (T*)a.v_pages + (slot * groups + h) * vp;
    for (int c = lane * VEC; c < vp; c += LANES * VEC) {
      float v[VEC];
#pragma unroll
      for (int e = 0; e < VEC; ++e) v[e] = 0.f;
      if (VEC > 1 || c < vdim) {
        load_vec<VEC>(src + c, v);
        if (bias) {
          float bv[VEC];
          load_vec<VEC>(bias + c, bv);
#pragma unroll
          for (int e = 0; e < VEC; ++e) v[e] += bv[e];
        }
      }
      store_vec<VEC>(dst + c, v);
    }
    return;
  }
  const int rot = (int)a.rot, half = rot / 2;
  int64_t pos = a.positions[t];
  pos = pos < 0 ? 0 : (pos < a.max_positions ? pos : a.max_positions - 1);
  const float* trig = a.cos_sin + pos * rot;
  const bool is_q = h < heads;
  const T* src = row + h * dim;
  T* dst = is_q ? (T*)a.q + (t * heads + h) * dp : (T*)a.k_pages + (slot * groups + h - heads) * dp;
  const T* w = (const T*)(is_q ? a.q_weight : a.k_weight);
  const T* bias = a.bias ? (const T*)a.bias + h * dim : nullptr;
  auto load = [&](int c, float (&v)[VEC]) {
    load_vec<VEC>(src + c, v);
    if (bias) {
      float bv[VEC];
      load_vec<VEC>(bias + c, bv);
#pragma unroll
      for (int e = 0; e < VEC; ++e) v[e] += bv[e];
    }
  };
  if (!is_q && !filed) return;
  if (VEC == 8) {
    const int c = lane * 8;
    const bool mine = c < dim, turns = c < rot, low = c < half;
    float v[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = 0.f;
    if (mine) load(c, v);
    float cs[VEC], sn[VEC];
    if (turns && !a.neighbours) {
      load_vec<VEC>(trig + (low ? c : c - half), cs);
      load_vec<VEC>(trig + half + (low ? c : c - half), sn);
    }
    if (w) {
      float ss = 0.f, wv[VEC];
      if (mine) load_vec<VEC>(w + c, wv);
#pragma unroll
      for (int e = 0; e < VEC; ++e) ss += v[e] * v[e];
      const float r = 1.0f / sqrtf(group_sum<LANES>(ss) / (float)dim + a.eps);
#pragma unroll
      for (int e = 0; e < VEC; ++e) v[e] = mine ? v[e] * r * wv[e] : 0.f;
    }
    if (a.neighbours) {      // whole pairs in a lane
      if (turns) {
        float pc[4], ps[4];
        load_vec<4>(trig + c / 2, pc);
        load_vec<4>(trig + half + c / 2, ps);
#pragma unroll
        for (int i = 0; i < VEC / 2; ++i) {
          const float x = v[2 * i], y = v[(2 * i + 1) % VEC];
          v[2 * i] = x * pc[i] - y * ps[i];
          v[(2 * i + 1) % VEC] = y * pc[i] + x * ps[i];
        }
      }
      if (mine) store_vec<VEC>(dst + c, v);
      return;
    }
    const int from = turns ? lane + (low ? half : -half) / 8 : lane;
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      const float o = __shfl(v[e], from, LANES);
      if (turns) v[e] = low ? v[e] * cs[e] - o * sn[e] : v[e] * cs[e] + o * sn[e];
    }
    if (mine) store_vec<VEC>(dst + c, v);
    return;
  }
  float r = 1.f;
  if (w) {
    float ss = 0.f;
    for (int c = lane * VEC; c < dim; c += LANES * VEC) {
      float v[VEC];
      load(c, v);
#pragma unroll
      for (int e = 0; e < VEC; ++e) ss += v[e] * v[e];
    }
    r = 1.0f / sqrtf(group_sum<LANES>(ss) / (float)dim + a.eps);
  }
  auto normed = [&](int c, float (&v)[VEC]) {
    load(c, v);
    if (w) {
      float wv[VEC];
      load_vec<VEC>(w + c, wv);
#pragma unroll
      for (int e = 0; e < VEC; ++e) v[e] = v[e] * r * wv[e];
    }
  };
  for (int c = lane * VEC; c < dp; c += LANES * VEC) {
    float v[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = 0.f;
    if (c < dim) {
      normed(c, v);
      if (c < rot) {
        const bool low = a.neighbours ? c % 2 == 0 : c < half;
        const int pair = a.neighbours ? c / 2 : (low ? c : c - half), mate = a.neighbours ? (low ? c + 1 : c - 1) : (low ? c + half : c - half);
        float o[VEC], cs[VEC], sn[VEC];
        normed(mate, o);
        load_vec<VEC>(trig + pair, cs);
        load_vec<VEC>(trig + half + pair, sn);
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] = low ? v[e] * cs[e] - o[e] * sn[e] : v[e] * cs[e] + o[e] * sn[e];
      }
    }
    store_vec<VEC>(dst + c, v);
  }
}

}  // namespace mops

extern "C" int mops_hip_rotary_prepare(const mops_hip_rotary_prepare_args* a, void* stream) {
  using namespace mops;
  if (!a || !known_dtype(a->dtype) || a->tokens < 0 || a->heads <= 0 || a->kv_heads <= 0 || a->dim <= 0 || a->vdim <= 0 || a->num_slots <= 0 ||
      a->max_positions <= 0 || a->rot < 0 || a->rot % 2 || a->rot > a->dim)
    return MOPS_HIP_EINVAL;
  if (a->tokens == 0) return MOPS_HIP_OK;
  if (!a->qkv || !a->positions || !a->slot_mapping || !a->q || !a->k_pages || !a->v_pages || (a->rot && !a->cos_sin)) return MOPS_HIP_EINVAL;
  if (a->qkv_stride < (a->heads + a->kv_heads) * a->dim + a->kv_heads * a->vdim) return MOPS_HIP_EINVAL;
  if (a->tokens > 0x7fffffffLL || a->heads * a->dim > (1 << 20) || a->kv_heads * (a->dim + a->vdim) > (1 << 20)) return MOPS_HIP_EUNSUPPORTED;
  const bool vec = a->dim % 8 == 0 && a->vdim % 8 == 0 && a->rot % (a->neighbours ? 8 : 16) == 0 && (!a->bias || aligned16(a->bias)) && a->qkv_stride % 8 == 0 && aligned16(a->qkv) && aligned16(a->q) &&
                   aligned16(a->k_pages) && aligned16(a->v_pages) && aligned16(a->cos_sin) && (!a->q_weight || aligned16(a->q_weight)) &&
                   (!a->k_weight || aligned16(a->k_weight));
  const int64_t items = a->heads + 2 * a->kv_heads, widest = a->dim > a->vdim ? a->dim : a->vdim;
  const bool wide = vec && widest <= 256;
  const int lanes = !wide ? 64 : (widest <= 64 ? 8 : (widest <= 128 ? 16 : 32));
  const int64_t wgs = (a->tokens * items + 256 / lanes - 1) / (256 / lanes);
  if (wgs > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  hipStream_t s = (hipStream_t)stream;
#define MOPS_RP(T, V, L) hipLaunchKernelGGL((rotary_prepare_kernel<T, V, L>), dim3((unsigned)wgs), dim3(256), 0, s, *a, (int)items)
#define MOPS_RP_TYPE(T) do {              \
    if (!wide) MOPS_RP(T, 1, 64);         \
    else if (lanes == 8) MOPS_RP(T, 8, 8);   \
    else if (lanes == 16) MOPS_RP(T, 8, 16); \
    else MOPS_RP(T, 8, 32);               \
  } while (0)
  if (a->dtype == MOPS_HIP_BF16) MOPS_RP_TYPE(bf16_t);
  else MOPS_RP_TYPE(float);
#undef MOPS_RP_TYPE
#undef MOPS_RP
  return finish_launch();
}
