// Mixture of experts: every token is sent to the `top` experts with the largest router logits.
//
//   moe_route    logits = router h in float32, the top choices per token, their sigmoid scores, and where each choice lands when
//                all choices are ordered by expert: row = (choices of earlier experts) + rank.  rows[] lists the choices (token *
//                top + place) by row; tiles[] cuts each expert's rows into blocks of `block_rows`.
//                Or the score is a choice's weight: experts are chosen by sigmoid + correction among those of the best groups of
//                neighbours, and the weights are their sigmoids over the sum of these, times a factor.
//   moe_gate_up  y[row] = silu(s W_gate h) * (s W_up h) with h the token's row and s its score: the score scales the expert's input;
//                or g sigmoid(alpha g) (u + 1) with g = min(W_gate h, limit), u = W_up h between -limit and limit
//   moe_down     z[choice] = W_down y[row], times the choice's weight in the second form
//   grouped_linear   the products of the small blocks without routing: equal runs of rows, each with weights of its own
// A unit that all tokens share can be part of both launches of the small blocks: workgroups of its own, which come first.
//
// The products are grouped: a workgroup takes a block of rows of one expert and some of its outputs.  Nothing comes back to the
// host: the grids are sized for the largest possible number of blocks, and workgroups without one leave.  The order of an
// expert's rows depends on the order in which the waves of a workgroup count them; no row's result depends on it.
//   large blocks   128 rows x 128 weight rows x 64 deep tiles through LDS, the next tile in flight into registers
//   small blocks   32 rows: weights are read once, straight into registers; the four waves split the depth
//   float          plain tiles on vector units
#include "mfma_tiles.h"

namespace mops {

constexpr int kMaxExperts = 1024;

struct RouteArgs {
  const void *h, *router;
  int64_t h_stride;
  int tokens, width, experts, top, per_wg;      // per_wg: tokens of a route workgroup, 16 or 32
  int32_t *chosen, *rank, *counts;     // [tokens * top], [tokens * top], [workgroups][experts]
  float* score;                        // [tokens * top]
  // the weighted form, with groups > 0
  const float* correction;             // [experts]
  int groups, keep;
  float factor;
};

// The weighted form, for LANES lanes per token (lane x owns the experts x, x + LANES, ...; N of them at most).  On entry score[e] is
// the sigmoid of expert e, choice[e] the same plus its correction, in LDS for all lanes of the token; group_score has room for the
// groups.  The lanes of a token run together: `together` orders their accesses to LDS.
template <int LANES, int N, typename Sync>
__device__ __forceinline__ void choose_weighted(const RouteArgs& a, const float* score, const float* choice, float* group_score, int x, int token, Sync together) {
  const int size = a.experts / a.groups;
  for (int g = x; g < a.groups; g += LANES) {      // the two best of a group
    float first = -INFINITY, second = -INFINITY;
    for (int e = g * size; e < (g + 1) * size; ++e) {
      const float c = choice[e];
      second = fmaxf(second, fminf(first, c));
      first = fmaxf(first, c);
    }
    group_score[g] = size > 1 ? first + second : first;
  }
  together();
  float mine[N];
  int place[N];
#pragma unroll
  for (int i = 0; i < N; ++i) {
    const int e = x + LANES * i;
    mine[i] = -INFINITY;
    place[i] = -1;
    if (e < a.experts) {
      bool open = a.keep >= a.groups;
      if (!open) {
        const int g = e / size;
        const float s = group_score[g];
        int better = 0;
        for (int o = 0; o < a.groups; ++o) better += group_score[o] > s || (group_score[o] == s && o < g);
        open = better < a.keep;
      }
      if (open) mine[i] = choice[e];
    }
  }
  float sum = 0.f;
  for (int s = 0; s < a.top; ++s) {
    float best = -INFINITY;
    int who = 0x7fffffff;
#pragma unroll
    for (int i = 0; i < N; ++i)
      if (mine[i] > best) {
        best = mine[i];
        who = x + LANES * i;
      }
#pragma unroll
    for (int off = 1; off < LANES; off <<= 1) {
      const float ob = __shfl_xor(best, off, kWave);
      const int ow = __shfl_xor(who, off, kWave);
      if (ob > best || (ob == best && ow < who)) {
        best = ob;
        who = ow;
      }
    }
    if (who >= a.experts) {      // scores that compare with nothing: any expert, and a weight that shows it
      if (x == 0 && token < a.tokens) {
        a.chosen[(int64_t)token * a.top + s] = s;
        a.score[(int64_t)token * a.top + s] = NAN;
      }
      continue;
    }
    sum += score[who];
#pragma unroll
    for (int i = 0; i < N; ++i)
      if (who == x + LANES * i) {
        mine[i] = -INFINITY;
        place[i] = s;
      }
  }
  const float f = a.factor / (sum + 1e-20f);
#pragma unroll
  for (int i = 0; i < N; ++i)
    if (place[i] >= 0 && token < a.tokens) {
      a.chosen[(int64_t)token * a.top + place[i]] = x + LANES * i;
      a.score[(int64_t)token * a.top + place[i]] = score[x + LANES * i] * f;
    }
}

constexpr int kPlaceGroups = 4;       // route workgroups of a place workgroup
// Tokens of a route workgroup: the router's weights are read once for all of them; small batches need the workgroups more.
static int route_tokens(int64_t tokens) { return tokens <= 2048 ? 16 : 32; }

// Counts this workgroup's choices per expert and ranks them among each other.
__device__ __forceinline__ void rank_choices(const RouteArgs& a, int* hist) {
  const int t0 = blockIdx.x * a.per_wg, n_tokens = a.tokens - t0 < a.per_wg ? a.tokens - t0 : a.per_wg;
  __syncthreads();
  for (int e = threadIdx.x; e < a.experts; e += 256) hist[e] = 0;
  __syncthreads();
  const int64_t i0 = (int64_t)t0 * a.top;
  for (int i = threadIdx.x; i < n_tokens * a.top; i += 256) a.rank[i0 + i] = atomicAdd(&hist[a.chosen[i0 + i]], 1);
  __syncthreads();
  for (int e = threadIdx.x; e < a.experts; e += 256) a.counts[(int64_t)blockIdx.x * a.experts + e] = hist[e];
}

// 16 TT tokens per workgroup on the matrix cores: bf16 operands, exact products, float32 sums; the four waves split the depth.
// ET: tiles of 16 experts.
template <int ET, int TT>
__global__ __launch_bounds__(256) void moe_route_mfma_kernel(const RouteArgs a, bool aligned) {
  constexpr int kPitch = ET * 16 + 1;
  constexpr int kAhead = TT == 1 ? (ET <= 2 ? 8 : (ET <= 4 ? 4 : 2)) : (ET <= 2 ? 4 : (ET <= 4 ? 2 : 1));      // steps whose loads are issued together
  __shared__ float logits[2][16 * TT][kPitch];
  __shared__ float group_scores[16 * TT][kPitch];
  __shared__ int hist[ET * 16];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, n = lane & 15, jj = lane >> 4;
  const int t0 = blockIdx.x * 16 * TT;
  const uint16_t *h[TT], *w[ET];
#pragma unroll
  for (int j = 0; j < TT; ++j) {
    const int t = t0 + 16 * j + n;
    h[j] = (const uint16_t*)a.h + (int64_t)(t < a.tokens ? t : a.tokens - 1) * a.h_stride;
  }
#pragma unroll
  for (int i = 0; i < ET; ++i) w[i] = (const uint16_t*)a.router + (int64_t)(16 * i + n < a.experts ? 16 * i + n : 0) * a.width;
  f32x4 acc[ET][TT];
#pragma unroll
  for (int i = 0; i < ET; ++i)
#pragma unroll
    for (int j = 0; j < TT; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 32 * kAhead * wave; k0 < a.width; k0 += 128 * kAhead) {
    u32x4 x[kAhead][TT], y[kAhead][ET];
#pragma unroll
    for (int s = 0; s < kAhead; ++s) {
      const int k = k0 + 32 * s + 8 * jj;
      if (aligned) {
        const bool ok = k < a.width;
#pragma unroll
        for (int j = 0; j < TT; ++j) {
          x[s][j] = load16(h[j] + (ok ? k : 0));
          if (!ok) x[s][j] = u32x4{0u, 0u, 0u, 0u};
        }
#pragma unroll
        for (int i = 0; i < ET; ++i) {
          y[s][i] = load16(w[i] + (ok ? k : 0));
          if (!ok) y[s][i] = u32x4{0u, 0u, 0u, 0u};
        }
      } else {
#pragma unroll
        for (int j = 0; j < TT; ++j) x[s][j] = load8_guarded(h[j], k, a.width, false);
#pragma unroll
        for (int i = 0; i < ET; ++i) y[s][i] = load8_guarded(w[i], k, a.width, false);
      }
    }
#pragma unroll
    for (int s = 0; s < kAhead; ++s)
#pragma unroll
      for (int i = 0; i < ET; ++i)
#pragma unroll
        for (int j = 0; j < TT; ++j) acc[i][j] = mfma16(__builtin_bit_cast(bf16x8, y[s][i]), __builtin_bit_cast(bf16x8, x[s][j]), acc[i][j]);
  }
  // the waves' parts: the first two leave theirs, the others add to them
#pragma unroll
  for (int round = 0; round < 2; ++round) {
    if (wave >> 1 == round) {
#pragma unroll
      for (int i = 0; i < ET; ++i)
#pragma unroll
        for (int j = 0; j < TT; ++j)
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            float& to = logits[wave & 1][16 * j + n][16 * i + 4 * jj + e];
            to = round ? to + acc[i][j][e] : acc[i][j][e];
          }
    }
    __syncthreads();
  }
  // sixteen lanes per token: lane x looks at the experts x, x + 16, ...
  const int x = threadIdx.x & 15;
#pragma unroll
  for (int j = 0; j < TT; ++j) {
    const int mt = 16 * j + (threadIdx.x >> 4), token = t0 + mt;
    if (a.groups > 0) {
      for (int e = x; e < a.experts; e += 16) {
        const float sg = 1.0f / (1.0f + expf(-(logits[0][mt][e] + logits[1][mt][e])));
        logits[0][mt][e] = sg + a.correction[e];
        logits[1][mt][e] = sg;
      }
      __syncthreads();
      choose_weighted<16, ET>(a, logits[1][mt], logits[0][mt], group_scores[mt], x, token, [] { __syncthreads(); });
      continue;
    }
    float mine[ET];
#pragma unroll
    for (int i = 0; i < ET; ++i) mine[i] = x + 16 * i < a.experts ? logits[0][mt][x + 16 * i] + logits[1][mt][x + 16 * i] : -INFINITY;
    for (int s = 0; s < a.top; ++s) {
      float best = -INFINITY;
      int who = 0x7fffffff;
#pragma unroll
      for (int i = 0; i < ET; ++i)
        if (mine[i] > best) {
          best = mine[i];
          who = x + 16 * i;
        }
#pragma unroll
      for (int off = 1; off < 16; off <<= 1) {
        const float ob = __shfl_xor(best, off, kWave);
        const int ow = __shfl_xor(who, off, kWave);
        if (ob > best || (ob == best && ow < who)) {
          best = ob;
          who = ow;
        }
      }
      if (who >= a.experts) {      // logits that compare with nothing: any expert that is left over, and a score that shows it
        who = s;
        best = NAN;
      }
#pragma unroll
      for (int i = 0; i < ET; ++i)
        if (who == x + 16 * i) mine[i] = -INFINITY;
      if (x == 0 && token < a.tokens) {
        a.chosen[(int64_t)token * a.top + s] = who;
        a.score[(int64_t)token * a.top + s] = 1.0f / (1.0f + expf(-best));
      }
    }
  }
  rank_choices(a, hist);
}

// A wave per token, any size.
template <typename T>
__global__ __launch_bounds__(256) void moe_route_kernel(const RouteArgs a) {
  __shared__ float logits[4][kMaxExperts], choices[4][kMaxExperts], group_scores[4][kMaxExperts];
  __shared__ int hist[kMaxExperts];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  float* mine = logits[wave];
  auto t0_of = [&](int i) { return (int)blockIdx.x * a.per_wg + i; };
  for (int i = wave; i < a.per_wg; i += 4) {      // as often for every wave
    const int t = t0_of(i);
    const T* h = (const T*)a.h + (int64_t)(t < a.tokens ? t : a.tokens - 1) * a.h_stride;
    for (int e = 0; e < a.experts; ++e) {
      const T* w = (const T*)a.router + (int64_t)e * a.width;
      float dot = 0.f;
      for (int k = lane; k < a.width; k += kWave) dot += to_f32(h[k]) * to_f32(w[k]);
      dot = group_sum<kWave>(dot);
      if (lane == 0) mine[e] = dot;
    }
    __syncthreads();
    if (a.groups > 0) {
      for (int e = lane; e < a.experts; e += kWave) {
        mine[e] = 1.0f / (1.0f + expf(-mine[e]));
        choices[wave][e] = mine[e] + a.correction[e];
      }
      __syncthreads();
      choose_weighted<kWave, kMaxExperts / kWave>(a, mine, choices[wave], group_scores[wave], lane, t0_of(i), [] { __syncthreads(); });
      __syncthreads();
      continue;
    }
    for (int s = 0; s < a.top; ++s) {
      float best = -INFINITY;
      int who = 0x7fffffff;
      for (int e = lane; e < a.experts; e += kWave)
        if (mine[e] > best) {
          best = mine[e];
          who = e;
        }
#pragma unroll
      for (int off = 1; off < 64; off <<= 1) {
        const float ob = __shfl_xor(best, off, kWave);
        const int ow = __shfl_xor(who, off, kWave);
        if (ob > best || (ob == best && ow < who)) {
          best = ob;
          who = ow;
        }
      }
      if (who >= a.experts) {
        who = s;
        best = NAN;
      }
      if ((who & 63) == lane) mine[who] = -INFINITY;      // the lane that looks at this expert
      if (lane == 0 && t < a.tokens) {
        a.chosen[(int64_t)t * a.top + s] = who;
        a.score[(int64_t)t * a.top + s] = 1.0f / (1.0f + expf(-best));
      }
    }
    __syncthreads();
  }
  rank_choices(a, hist);
}

// rows[] and tiles[]; a workgroup for every kPlaceGroups of the route.  tiles: [0] their number, then {expert, first row, rows} each.
__global__ __launch_bounds__(256) void moe_place_kernel(const RouteArgs a, int groups, int32_t* __restrict__ rows, int32_t* __restrict__ tiles, int block_rows) {
  __shared__ int total[kMaxExperts], earlier[kMaxExperts];
  __shared__ int begin[kMaxExperts + 1], first_tile[kMaxExperts + 1];
  __shared__ int wave_rows[4], wave_tiles[4];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  for (int e = tid; e < kMaxExperts; e += 256) total[e] = earlier[e] = 0;
  __syncthreads();
  {
    // threads over (experts, part of the workgroups); four experts at a time where rows of counts are aligned
    const int mine = blockIdx.x * kPlaceGroups, step = a.experts % 4 == 0 ? 4 : 1, columns = a.experts / step;
    const int across = columns < 256 ? columns : 256, parts = 256 / across;
    if (tid < across * parts)
      for (int c = tid % across; c < columns; c += across) {
        int all[4] = {0, 0, 0, 0}, front[4] = {0, 0, 0, 0};
        if (step == 4) {
#pragma unroll 4
          for (int w = tid / across; w < groups; w += parts) {
            const u32x4 v = load16(a.counts + (int64_t)w * a.experts + 4 * c);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              all[e] += (int)v[e];
              front[e] += w < mine ? (int)v[e] : 0;
            }
          }
        } else {
#pragma unroll 8
          for (int w = tid / across; w < groups; w += parts) {
            const int v = a.counts[(int64_t)w * a.experts + c];
            all[0] += v;
            front[0] += w < mine ? v : 0;
          }
        }
        for (int e = 0; e < step; ++e) {
          atomicAdd(&total[c * step + e], all[e]);
          atomicAdd(&earlier[c * step + e], front[e]);
        }
      }
  }
  __syncthreads();
  {
    // a thread owns four consecutive experts
    int c[4], r = 0, n = 0;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      c[i] = total[4 * tid + i];
      r += c[i];
      n += (c[i] + block_rows - 1) / block_rows;
    }
    int ri = r, ni = n;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const int ru = __shfl_up(ri, off, 64), nu = __shfl_up(ni, off, 64);
      if (lane >= off) {
        ri += ru;
        ni += nu;
      }
    }
    if (lane == 63) {
      wave_rows[wave] = ri;
      wave_tiles[wave] = ni;
    }
    __syncthreads();
    r = ri - r;
    n = ni - n;
    for (int w = 0; w < wave; ++w) {
      r += wave_rows[w];
      n += wave_tiles[w];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      begin[4 * tid + i] = r;
      first_tile[4 * tid + i] = n;
      r += c[i];
      n += (c[i] + block_rows - 1) / block_rows;
    }
    if (tid == 255) {
      begin[kMaxExperts] = r;
      first_tile[kMaxExperts] = n;
    }
  }
  __syncthreads();
  const int per = a.per_wg * kPlaceGroups, t0 = blockIdx.x * per, n_tokens = a.tokens - t0 < per ? a.tokens - t0 : per;
  for (int i = tid; i < n_tokens * a.top; i += 256) {
    const int choice = t0 * a.top + i, e = a.chosen[choice];
    int at = begin[e] + earlier[e] + a.rank[choice];
    for (int w = blockIdx.x * kPlaceGroups; w < choice / a.top / a.per_wg; ++w) at += a.counts[(int64_t)w * a.experts + e];
    rows[at] = choice;
  }
  if (blockIdx.x == 0) {
    if (tid == 0) tiles[0] = first_tile[kMaxExperts];
    for (int e = tid; e < a.experts; e += 256)
      for (int r = begin[e], k = first_tile[e]; r < begin[e + 1]; r += block_rows, ++k) {
        tiles[1 + 3 * k] = e;
        tiles[2 + 3 * k] = r;
        tiles[3 + 3 * k] = begin[e + 1] - r < block_rows ? begin[e + 1] - r : block_rows;
      }
  }
}

struct GroupedArgs {
  const void* x;            // gate_up: h [tokens, x_stride]; down: y [rows, x_stride]
  int64_t x_stride;
  const void* w;            // [experts][w_rows][depth]
  int64_t w_expert;         // elements per expert
  int n, up_at, depth;      // outputs, first up row behind the gate rows, depth of the product
  void* out;
  int64_t out_stride;
  const int32_t *rows, *tiles;
  const float* score;
  int top, blocks;          // blocks of outputs in the grid
  int unit;                 // of gate_up: 0 silu of scaled inputs, 1 clamped
  float limit, alpha;
  bool weigh;               // the choice's score multiplies the result of down instead of the input of gate_up
  // small blocks without routing (rows == nullptr): group e has the rows e * per_group .., and one more group of the same rows has
  // weights, outputs and their number of its own
  int per_group, groups;
  const void* w_last;
  int n_last;
  void* out_last;
  int64_t out_last_stride;
  // small blocks with a shared unit: the first `ahead` workgroups (a multiple of 8); its rows are the tokens, and more is its own
  int ahead, tokens;
  const void* x_last;
  int64_t x_last_stride;
  int up_last, depth_last;
  float limit_last;
};

// The gated unit of an expert: s the choice's score, g and u the products of its token.
template <typename T>
__device__ __forceinline__ float gated_unit(const GroupedArgs& a, float limit, float s, float g, float u) {
  if (a.unit == 0) return silu_for<T>(s * g) * (s * u);
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * sigmoid_for<T>(a.alpha * g) * (u + 1.0f);
}

// This workgroup's tile and block of outputs.  Consecutive workgroups go to different XCDs: each XCD gets a contiguous run of
// tiles with all their outputs, so that the rows of a tile and the weights of an expert meet in one L2.
__device__ __forceinline__ bool grouped_item(const GroupedArgs& a, int& tile, int& block) {
  const int n = a.tiles[0], per = (n + 7) / 8, i = ((int)blockIdx.x - a.ahead) / 8;
  tile = (blockIdx.x % 8) * per + i / a.blocks;
  block = i % a.blocks;
  return i / a.blocks < per && tile < n;
}

// ---------------------------------------------------------------------------------------------------- large blocks
constexpr int kGM = 128, kGK = 64, kGPitch = kGK + 8, kGTile = 128 * kGPitch;

template <bool GATED, bool ALIGNED>
__global__ __launch_bounds__(256, 2) void moe_grouped_large_kernel(const GroupedArgs a) {
  extern __shared__ __align__(16) unsigned char smem[];
  uint16_t* const lds = reinterpret_cast<uint16_t*>(smem);      // two buffers of [x tile | w tile]
  int tile, block;
  if (!grouped_item(a, tile, block)) return;
  const int e = a.tiles[1 + 3 * tile], row0 = a.tiles[2 + 3 * tile], count = a.tiles[3 + 3 * tile];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 31, hh = lane >> 5;
  const int wm = wave & 1, wn = wave >> 1;
  constexpr int kOut = GATED ? 64 : 128;                         // outputs of the workgroup
  const int n0 = block * kOut;
  const uint16_t* w = (const uint16_t*)a.w + (int64_t)e * a.w_expert;
  // pieces of 16 bytes: thread -> row tid / 8 + 32 j, depth 8 (tid % 8)
  const int prow = tid >> 3, pk = (tid & 7) * 8;
  const uint16_t *xp[4], *wp[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int r = prow + 32 * j;
    const int src = row0 + (r < count ? r : count - 1);
    xp[j] = (const uint16_t*)a.x + (int64_t)(GATED ? a.rows[src] / a.top : src) * a.x_stride;
    const int n = GATED ? (r < 64 ? n0 + r : n0 + r - 64) : n0 + r;
    wp[j] = w + (int64_t)((n < a.n ? n : 0) + (GATED && r >= 64 ? a.up_at : 0)) * a.depth;
  }
  // Loads carry no condition: behind the depth they read the row's start, and the pieces become zeros on their way into LDS.
  u32x4 xr[2][4], wr[2][4];
  auto issue = [&](u32x4 (&x)[4], u32x4 (&y)[4], int k0) {
    const int k = k0 + pk, at = k < a.depth ? k : 0;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      x[j] = ALIGNED ? load16(xp[j] + at) : load8_guarded(xp[j], k, a.depth, false);
      y[j] = ALIGNED ? load16(wp[j] + at) : load8_guarded(wp[j], k, a.depth, false);
    }
  };
  auto stash = [&](const u32x4 (&x)[4], const u32x4 (&y)[4], int buf, int k0) {
    uint16_t* d = lds + buf * 2 * kGTile + prow * kGPitch + pk;
    const bool ok = k0 + pk < a.depth;
    const u32x4 zero = {0u, 0u, 0u, 0u};
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      store16(d + 32 * j * kGPitch, ok ? x[j] : zero);
      store16(d + kGTile + 32 * j * kGPitch, ok ? y[j] : zero);
    }
  };
  f32x16 acc[2][2];      // [weight rows][tokens]
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[i][j][r] = 0.f;
  auto multiply = [&](int buf) {
    const uint16_t *tx = lds + buf * 2 * kGTile, *tw = tx + kGTile;
#pragma unroll
    for (int kk = 0; kk < kGK / 16; ++kk) {
      bf16x8 wf[2], xf[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) wf[i] = tile_row(tw, kGPitch, (GATED ? 64 * i + 32 * wn : 64 * wn + 32 * i) + col, 16 * kk + 8 * hh);
#pragma unroll
      for (int j = 0; j < 2; ++j) xf[j] = tile_row(tx, kGPitch, 64 * wm + 32 * j + col, 16 * kk + 8 * hh);
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i][j] = mfma32(wf[i], xf[j], acc[i][j]);
    }
  };
  // a turn: two tiles, each with the loads of the tile two further on issued in front of its products
  issue(xr[0], wr[0], 0);
  issue(xr[1], wr[1], kGK);
  stash(xr[0], wr[0], 0, 0);
  __syncthreads();
  for (int k0 = 0; k0 < a.depth; k0 += 2 * kGK) {
    issue(xr[0], wr[0], k0 + 2 * kGK);
    multiply(0);
    if (k0 + kGK >= a.depth) break;
    stash(xr[1], wr[1], 1, k0 + kGK);
    __syncthreads();
    issue(xr[1], wr[1], k0 + 3 * kGK);
    multiply(1);
    if (k0 + 2 * kGK >= a.depth) break;
    stash(xr[0], wr[0], 0, k0 + 2 * kGK);
    __syncthreads();
  }
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int r = 64 * wm + 32 * j + col;
    if (r >= count) continue;
    const int choice = a.rows[row0 + r];
    const float s = GATED != a.weigh ? a.score[choice] : 1.f;
    uint16_t* o = (uint16_t*)a.out + (int64_t)(GATED ? row0 + r : choice) * a.out_stride;
#pragma unroll
    for (int i = 0; i < (GATED ? 1 : 2); ++i)
#pragma unroll
      for (int q4 = 0; q4 < 4; ++q4) {
        const int n = n0 + (GATED ? 32 * wn : 64 * wn + 32 * i) + 8 * q4 + 4 * hh;
        float v[4];
#pragma unroll
        for (int x = 0; x < 4; ++x) v[x] = GATED ? gated_unit<bf16_t>(a, a.limit, s, acc[0][j][4 * q4 + x], acc[1][j][4 * q4 + x]) : s * acc[i][j][4 * q4 + x];
        if (ALIGNED && n + 4 <= a.n) {
          *reinterpret_cast<u32x2*>(o + n) = u32x2{pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3])};
        } else {
#pragma unroll
          for (int x = 0; x < 4; ++x)
            if (n + x < a.n) o[n + x] = (uint16_t)f32_to_bf16_bits(v[x]);
        }
      }
  }
}

// ---------------------------------------------------------------------------------------------------- small blocks
constexpr int kSM = 32;

// Four 16-row pieces of the weights: GATED two of gate rows and two of up rows (32 outputs), else 64 outputs; two pieces of 16 rows.
template <bool GATED, bool ALIGNED>
__global__ __launch_bounds__(256, 3) void moe_grouped_small_kernel(const GroupedArgs a) {
  __shared__ __align__(16) f32x4 part[4][8][64];      // [wave][piece of the weights, piece of the rows][lane]
  int tile, block;
  int e, row0, count, n_all = a.n;
  int depth = a.depth, up_at = a.up_at;
  float limit = a.limit;
  const uint16_t *w_group, *xs = (const uint16_t*)a.x;
  int64_t x_stride = a.x_stride;
  bool last = false;
  const bool common = a.tiles && (int)blockIdx.x < a.ahead;
  if (common) {
    // each XCD takes every eighth block of weights, with all row tiles
    const int per = (a.tokens + kSM - 1) / kSM, c = (int)blockIdx.x;
    tile = c / 8 % per;
    block = c % 8 + 8 * (c / 8 / per);
    e = 0;
    row0 = tile * kSM;
    count = a.tokens - row0 < kSM ? a.tokens - row0 : kSM;
    last = true;
    n_all = a.n_last;
    w_group = (const uint16_t*)a.w_last;
    xs = (const uint16_t*)a.x_last;
    x_stride = a.x_last_stride;
    depth = a.depth_last;
    up_at = a.up_last;
    limit = a.limit_last;
    if (block * (GATED ? 32 : 64) >= n_all) return;
  } else if (a.tiles) {
    if (!grouped_item(a, tile, block)) return;
    e = a.tiles[1 + 3 * tile];
    row0 = a.tiles[2 + 3 * tile];
    count = a.tiles[3 + 3 * tile];
    w_group = (const uint16_t*)a.w + (int64_t)e * a.w_expert;
  } else {
    // all row tiles of a block of weights one behind the other
    const int per = (a.per_group + kSM - 1) / kSM;
    tile = blockIdx.x % per;
    block = blockIdx.x / per % a.blocks;
    e = blockIdx.x / per / a.blocks;
    row0 = e * a.per_group + tile * kSM;
    count = a.per_group - tile * kSM < kSM ? a.per_group - tile * kSM : kSM;
    last = e == a.groups;
    n_all = last ? a.n_last : a.n;
    w_group = last ? (const uint16_t*)a.w_last : (const uint16_t*)a.w + (int64_t)e * a.w_expert;
    if (block * 64 >= n_all) return;
  }
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 15, jj = lane >> 4;
  const int n0 = block * (GATED ? 32 : 64);
  const uint16_t *x[2], *w[4];
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int r = 16 * j + col, src = row0 + (r < count ? r : count - 1);
    x[j] = xs + (int64_t)(GATED && !common ? a.rows[src] / a.top : src) * x_stride;
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int n = n0 + 16 * (GATED ? i & 1 : i) + col;      // outputs behind the last are row 0 again and never stored
    w[i] = w_group + (int64_t)((n < n_all ? n : 0) + (GATED && i >= 2 ? up_at : 0)) * depth;
  }
  f32x4 acc[4][2];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  // a wave takes every fourth piece of 32 of the depth, with two pieces in flight while one is used
  u32x4 xr[3][2], wr[3][4];
  const int pieces = (depth - 32 * wave + 127) / 128;
  auto fetch = [&](int buf, int piece) {
    const int k = 32 * wave + 128 * piece + 8 * jj;
    if (ALIGNED) {
      const bool ok = k < depth;
#pragma unroll
      for (int i = 0; i < 4; ++i) wr[buf][i] = load16(w[i] + (ok ? k : 0));
#pragma unroll
      for (int j = 0; j < 2; ++j) xr[buf][j] = load16(x[j] + (ok ? k : 0));
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i) wr[buf][i] = load8_guarded(w[i], k, depth, false);
#pragma unroll
      for (int j = 0; j < 2; ++j) xr[buf][j] = load8_guarded(x[j], k, depth, false);
    }
  };
  auto use = [&](int buf, int piece) {
    const bool ok = 32 * wave + 128 * piece + 8 * jj < depth;      // what lies behind the depth counts as zeros on both sides
    const u32x4 zero = {0u, 0u, 0u, 0u};
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const bf16x8 b = __builtin_bit_cast(bf16x8, ok ? xr[buf][j] : zero);
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[i][j] = mfma16(__builtin_bit_cast(bf16x8, ok ? wr[buf][i] : zero), b, acc[i][j]);
    }
  };
  if (pieces > 0) {
    fetch(0, 0);
    fetch(1, 1);
    for (int p = 0;; p += 3) {      // three pieces a turn: the buffers are registers
      fetch(2, p + 2);
      use(0, p);
      if (p + 1 >= pieces) break;
      fetch(0, p + 3);
      use(1, p + 1);
      if (p + 2 >= pieces) break;
      fetch(1, p + 4);
      use(2, p + 2);
      if (p + 3 >= pieces) break;
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) part[wave][2 * i + j][lane] = acc[i][j];
  __syncthreads();
  // wave (i, j): rows 16 j .., outputs of the pieces i (and i + 2)
  const int i = wave >> 1, j = wave & 1, r = 16 * j + col;
  auto total = [&](int piece) { return (part[0][piece][lane] + part[1][piece][lane]) + (part[2][piece][lane] + part[3][piece][lane]); };
  const f32x4 v0 = total(2 * i + j), v1 = total(2 * (i + 2) + j);
  if (r >= count) return;
  const int choice = a.rows && !common ? a.rows[row0 + r] : row0 + r;
  uint16_t* o = last ? (uint16_t*)a.out_last + (int64_t)(choice - e * a.per_group) * a.out_last_stride
                     : (uint16_t*)a.out + (int64_t)(GATED ? row0 + r : choice) * a.out_stride;
  const float s = GATED != a.weigh && !common ? a.score[choice] : 1.f;
#pragma unroll
  for (int half = 0; half < (GATED ? 1 : 2); ++half) {
    const int n = n0 + 16 * (i + 2 * half) + 4 * jj;
    float y[4];
#pragma unroll
    for (int q = 0; q < 4; ++q) y[q] = GATED ? gated_unit<bf16_t>(a, limit, s, v0[q], v1[q]) : s * (half ? v1[q] : v0[q]);
    if (ALIGNED && n + 4 <= n_all) {
      *reinterpret_cast<u32x2*>(o + n) = u32x2{pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3])};
    } else {
#pragma unroll
      for (int q = 0; q < 4; ++q)
        if (n + q < n_all) o[n + q] = (uint16_t)f32_to_bf16_bits(y[q]);
    }
  }
}

// ---------------------------------------------------------------------------------------------------- float
// 32 rows x 64 outputs per workgroup; a thread takes one output of eight rows.
template <bool GATED>
__global__ __launch_bounds__(256) void moe_grouped_f32_kernel(const GroupedArgs a) {
  __shared__ float tx[kSM][33], tw[GATED ? 2 : 1][64][33];
  int tile, block;
  if (!grouped_item(a, tile, block)) return;
  const int e = a.tiles[1 + 3 * tile], row0 = a.tiles[2 + 3 * tile], count = a.tiles[3 + 3 * tile];
  const int tid = threadIdx.x, n_loc = tid & 63, r0 = tid >> 6;
  const int n0 = block * 64;
  const float* w = (const float*)a.w + (int64_t)e * a.w_expert;
  float acc[GATED ? 2 : 1][8];
#pragma unroll
  for (int i = 0; i < (GATED ? 2 : 1); ++i)
#pragma unroll
    for (int r = 0; r < 8; ++r) acc[i][r] = 0.f;
  for (int k0 = 0; k0 < a.depth; k0 += 32) {
    for (int i = tid; i < kSM * 32; i += 256) {
      const int r = i / 32, k = k0 + i % 32;
      const int src = row0 + (r < count ? r : count - 1);
      tx[r][i % 32] = k < a.depth ? ((const float*)a.x)[(int64_t)(GATED ? a.rows[src] / a.top : src) * a.x_stride + k] : 0.f;
    }
    for (int i = tid; i < (GATED ? 2 : 1) * 64 * 32; i += 256) {
      const int half = i / (64 * 32), r = i / 32 % 64, k = k0 + i % 32;
      tw[half][r][i % 32] = k < a.depth && n0 + r < a.n ? w[(int64_t)(n0 + r + (half ? a.up_at : 0)) * a.depth + k] : 0.f;
    }
    __syncthreads();
    for (int k = 0; k < 32; ++k)
#pragma unroll
      for (int i = 0; i < (GATED ? 2 : 1); ++i)
#pragma unroll
        for (int r = 0; r < 8; ++r) acc[i][r] += tw[i][n_loc][k] * tx[r0 + 4 * r][k];
    __syncthreads();
  }
  const int n = n0 + n_loc;
  if (n >= a.n) return;
#pragma unroll
  for (int r = 0; r < 8; ++r) {
    const int row = r0 + 4 * r;
    if (row >= count) continue;
    const int choice = a.rows[row0 + row];
    const float s = GATED != a.weigh ? a.score[choice] : 1.f;
    ((float*)a.out)[(int64_t)(GATED ? row0 + row : choice) * a.out_stride + n] =
        GATED ? gated_unit<float>(a, a.limit, s, acc[0][r], acc[GATED ? 1 : 0][r]) : s * acc[0][r];
  }
}

template <bool GATED>
static int launch_grouped(GroupedArgs a, int dtype, int64_t block_rows, int64_t choices, int64_t experts, hipStream_t s) {
  const int64_t tiles = choices / block_rows + (experts < choices ? experts : choices);
  const int per = dtype == MOPS_HIP_F32 ? 64 : (block_rows == kSM ? (GATED ? 32 : 64) : (GATED ? 64 : 128));
  a.blocks = (a.n + per - 1) / per;
  int64_t grid_size = (tiles + 7) / 8 * 8 * a.blocks;
  const int64_t ahead = a.w_last ? (int64_t)((a.n_last + per - 1) / per + 7) / 8 * 8 * ((a.tokens + kSM - 1) / kSM) : 0;
  a.ahead = (int)(ahead < 0x7fffffffLL ? ahead : 0x7fffffffLL);
  grid_size += ahead;
  if (grid_size > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  const dim3 grid((unsigned)grid_size), block(256);
  const bool aligned = a.depth % 8 == 0 && a.x_stride % 8 == 0 && a.out_stride % 4 == 0 && a.w_expert % 8 == 0 && aligned16(a.x) && aligned16(a.w) &&
                       aligned16(a.out) &&
                       (!a.w_last || (a.depth_last % 8 == 0 && a.x_last_stride % 8 == 0 && a.out_last_stride % 4 == 0 && aligned16(a.x_last) &&
                                      aligned16(a.w_last) && aligned16(a.out_last)));
  if (dtype == MOPS_HIP_F32) {
    hipLaunchKernelGGL((moe_grouped_f32_kernel<GATED>), grid, block, 0, s, a);
  } else if (block_rows == kSM) {
    if (aligned) hipLaunchKernelGGL((moe_grouped_small_kernel<GATED, true>), grid, block, 0, s, a);
    else hipLaunchKernelGGL((moe_grouped_small_kernel<GATED, false>), grid, block, 0, s, a);
  } else {
    constexpr int kLds = 4 * kGTile * 2;
    static const hipError_t lds0 = hipFuncSetAttribute(reinterpret_cast<const void*>(&moe_grouped_large_kernel<GATED, true>),
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, kLds);
    static const hipError_t lds1 = hipFuncSetAttribute(reinterpret_cast<const void*>(&moe_grouped_large_kernel<GATED, false>),
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, kLds);
    if (lds0 != hipSuccess) return record_hip_error(lds0);
    if (lds1 != hipSuccess) return record_hip_error(lds1);
    if (aligned) hipLaunchKernelGGL((moe_grouped_large_kernel<GATED, true>), grid, block, kLds, s, a);
    else hipLaunchKernelGGL((moe_grouped_large_kernel<GATED, false>), grid, block, kLds, s, a);
  }
  return finish_launch();
}

static int check_grouped(const mops_hip_moe* m) {
  if (!m || !known_dtype(m->dtype) || m->tokens < 0) return MOPS_HIP_EINVAL;
  if (m->tokens == 0) return MOPS_HIP_OK;
  if (m->experts <= 0 || m->top <= 0 || m->top > m->experts || m->width <= 0 || m->ff <= 0) return MOPS_HIP_EINVAL;
  if (m->block_rows != kSM && (m->block_rows != kGM || m->dtype != MOPS_HIP_BF16)) return MOPS_HIP_EINVAL;
  if (m->experts > kMaxExperts || m->tokens * m->top > (1 << 28) || m->width > (1 << 20) || m->ff > (1 << 20)) return MOPS_HIP_EUNSUPPORTED;
  if (!m->rows || !m->tiles || !m->score) return MOPS_HIP_EINVAL;
  if (m->groups < 0 || (m->groups > 0 && (m->experts % m->groups || m->keep <= 0 || m->keep > m->groups || m->top > m->experts / m->groups * m->keep)))
    return MOPS_HIP_EINVAL;
  if (m->unit != 0 && m->unit != 1) return MOPS_HIP_EINVAL;
  if (m->common_w) {
    if (m->block_rows != kSM || m->dtype != MOPS_HIP_BF16 || !m->common_x || !m->common_out || m->common_ff <= 0) return MOPS_HIP_EINVAL;
    if (m->common_ff > (1 << 20) || m->common_up_at > (1 << 20)) return MOPS_HIP_EUNSUPPORTED;
  }
  return 1;
}

// What both launches say about the shared unit.
static void set_common(GroupedArgs& a, const mops_hip_moe* m) {
  a.w_last = m->common_w;
  a.x_last = m->common_x;
  a.out_last = m->common_out;
  a.x_last_stride = m->common_x_stride;
  a.out_last_stride = m->common_out_stride;
  a.limit_last = m->common_limit;
  a.tokens = (int)m->tokens;
}

}  // namespace mops

extern "C" int64_t mops_hip_moe_max_tiles(int64_t tokens, int64_t experts, int64_t top, int64_t block_rows) {
  if (tokens < 0 || experts <= 0 || top <= 0 || block_rows <= 0) return MOPS_HIP_EINVAL;
  const int64_t choices = tokens * top;
  return choices / block_rows + (experts < choices ? experts : choices);
}

extern "C" int64_t mops_hip_moe_route_workgroups(int64_t tokens) {
  if (tokens < 0) return MOPS_HIP_EINVAL;
  return (tokens + mops::route_tokens(tokens) - 1) / mops::route_tokens(tokens);
}

extern "C" int mops_hip_moe_route(const void* h, int64_t h_row_stride, const void* router, int32_t* chosen, int32_t* rank, int32_t* counts,
                                  const mops_hip_moe* m, void* stream) {
  using namespace mops;
  const int pre = check_grouped(m);
  if (pre != 1) return pre;
  if (!h || !router || !chosen || !rank || !counts || h_row_stride < m->width) return MOPS_HIP_EINVAL;
  if (!aligned16(counts)) return MOPS_HIP_EALIGN;
  RouteArgs a;
  a.h = h; a.router = router; a.h_stride = h_row_stride;
  a.tokens = (int)m->tokens; a.width = (int)m->width; a.experts = (int)m->experts; a.top = (int)m->top;
  a.chosen = chosen; a.rank = rank; a.counts = counts; a.score = m->score;
  a.per_wg = route_tokens(m->tokens);
  if (m->groups > 0 && !m->correction) return MOPS_HIP_EINVAL;
  a.correction = m->correction; a.groups = (int)m->groups; a.keep = (int)m->keep; a.factor = m->factor;
  const int64_t groups = mops_hip_moe_route_workgroups(m->tokens);
  const dim3 grid((unsigned)groups), block(256);
  hipStream_t s = (hipStream_t)stream;
  if (m->dtype == MOPS_HIP_BF16 && m->experts <= 128) {
    const bool aligned = m->width % 8 == 0 && h_row_stride % 8 == 0 && aligned16(h) && aligned16(router);
#define MOPS_ROUTE(E) do {                                                                                                \
    if (a.per_wg == 16) hipLaunchKernelGGL((moe_route_mfma_kernel<E, 1>), grid, block, 0, s, a, aligned);                \
    else hipLaunchKernelGGL((moe_route_mfma_kernel<E, 2>), grid, block, 0, s, a, aligned);                               \
  } while (0)
    if (m->experts <= 16) MOPS_ROUTE(1);
    else if (m->experts <= 32) MOPS_ROUTE(2);
    else if (m->experts <= 64) MOPS_ROUTE(4);
    else MOPS_ROUTE(8);
#undef MOPS_ROUTE
  } else if (m->dtype == MOPS_HIP_BF16) {
    hipLaunchKernelGGL((moe_route_kernel<bf16_t>), grid, block, 0, s, a);
  } else {
    hipLaunchKernelGGL((moe_route_kernel<float>), grid, block, 0, s, a);
  }
  int st = finish_launch();
  if (st != MOPS_HIP_OK) return st;
  hipLaunchKernelGGL(moe_place_kernel, dim3((unsigned)((groups + kPlaceGroups - 1) / kPlaceGroups)), block, 0, s, a, (int)groups, m->rows, m->tiles, (int)m->block_rows);
  return finish_launch();
}

extern "C" int mops_hip_moe_gate_up(const void* h, int64_t h_row_stride, const void* w, int64_t up_at, void* y, int64_t y_row_stride,
                                    const mops_hip_moe* m, void* stream) {
  using namespace mops;
  const int pre = check_grouped(m);
  if (pre != 1) return pre;
  if (!h || !w || !y || h_row_stride < m->width || y_row_stride < m->ff || up_at < m->ff || up_at > (1 << 20)) return MOPS_HIP_EINVAL;
  GroupedArgs a = {};
  a.x = h; a.x_stride = h_row_stride; a.w = w; a.w_expert = 2 * up_at * m->width;
  a.n = (int)m->ff; a.up_at = (int)up_at; a.depth = (int)m->width; a.out = y; a.out_stride = y_row_stride;
  a.rows = m->rows; a.tiles = m->tiles; a.score = m->score; a.top = (int)m->top; a.blocks = 0;
  a.unit = m->unit; a.limit = m->limit; a.alpha = m->alpha; a.weigh = m->groups > 0;
  if (m->common_w) {
    if (m->unit != 1 || m->common_up_at < m->common_ff || m->common_x_stride < m->width || m->common_out_stride < m->common_ff) return MOPS_HIP_EINVAL;
    set_common(a, m);
    a.n_last = (int)m->common_ff; a.up_last = (int)m->common_up_at; a.depth_last = (int)m->width;
  }
  return launch_grouped<true>(a, m->dtype, m->block_rows, m->tokens * m->top, m->experts, (hipStream_t)stream);
}

extern "C" int mops_hip_moe_down(const void* y, int64_t y_row_stride, const void* w, int64_t depth, void* z, int64_t z_row_stride,
                                 const mops_hip_moe* m, void* stream) {
  using namespace mops;
  const int pre = check_grouped(m);
  if (pre != 1) return pre;
  if (!y || !w || !z || depth < m->ff || depth > (1 << 20) || y_row_stride < depth || z_row_stride < m->width) return MOPS_HIP_EINVAL;
  GroupedArgs a = {};
  a.x = y; a.x_stride = y_row_stride; a.w = w; a.w_expert = depth * m->width;
  a.n = (int)m->width; a.up_at = 0; a.depth = (int)depth; a.out = z; a.out_stride = z_row_stride;
  a.rows = m->rows; a.tiles = m->tiles; a.score = m->score; a.top = (int)m->top; a.blocks = 0; a.weigh = m->groups > 0;
  if (m->common_w) {
    if (m->common_x_stride < m->common_ff || m->common_out_stride < m->width) return MOPS_HIP_EINVAL;
    set_common(a, m);
    a.n_last = (int)m->width; a.depth_last = (int)m->common_ff;
  }
  return launch_grouped<false>(a, m->dtype, m->block_rows, m->tokens * m->top, m->experts, (hipStream_t)stream);
}

extern "C" int mops_hip_grouped_linear(const void* x, const void* w, void* y, const void* w_last, void* y_last, int64_t n_last, int64_t groups,
                                       int64_t tokens, int64_t n, int64_t k, void* stream) {
  using namespace mops;
  if (groups <= 0 || tokens < 0 || n <= 0 || k <= 0 || (w_last && (!y_last || n_last <= 0 || n_last > n))) return MOPS_HIP_EINVAL;
  if (tokens == 0) return MOPS_HIP_OK;
  if (!x || !w || !y) return MOPS_HIP_EINVAL;
  if (n > (1 << 20) || k > (1 << 20) || (groups + 1) * tokens > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  GroupedArgs a = {};
  a.x = x; a.x_stride = k; a.w = w; a.w_expert = n * k; a.n = (int)n; a.depth = (int)k; a.out = y; a.out_stride = n; a.top = 1;
  a.blocks = (int)((n + 63) / 64);
  a.per_group = (int)tokens; a.groups = (int)groups; a.w_last = w_last; a.n_last = (int)n_last; a.out_last = y_last; a.out_last_stride = n_last;
  const int64_t grid = (tokens + kSM - 1) / kSM * a.blocks * (groups + (w_last ? 1 : 0));
  if (grid > 0x7fffffffLL) return MOPS_HIP_EUNSUPPORTED;
  const bool aligned = k % 8 == 0 && n % 4 == 0 && aligned16(x) && aligned16(w) && aligned16(y) &&
                       (!w_last || (n_last % 4 == 0 && aligned16(w_last) && aligned16(y_last)));
  if (aligned) hipLaunchKernelGGL((moe_grouped_small_kernel<false, true>), dim3((unsigned)grid), dim3(256), 0, (hipStream_t)stream, a);
  else hipLaunchKernelGGL((moe_grouped_small_kernel<false, false>), dim3((unsigned)grid), dim3(256), 0, (hipStream_t)stream, a);
  return finish_launch();
}
