// Which tokens of its sequence a query row sees.
#pragma once
#include "mixed_types.h"

namespace mops {

constexpr int kMaxRange = 1 << 30;      // windows, chunks and counts of kept tokens stay below it

// Tokens lo .. and 0 .. kept-1 (kept <= lo), up to the row's own position.
struct Visible { int lo, kept; };

__device__ __forceinline__ int first_visible(const mops_hip_biased_attention& a, int pos) {
  if (a.window > 0) return pos >= (int)a.window ? pos - (int)a.window + 1 : 0;
  return a.chunk > 0 ? pos / (int)a.chunk * (int)a.chunk : 0;
}
__device__ __forceinline__ Visible visible_at(const mops_hip_biased_attention& a, int len) {
  const int lo = len > 0 ? first_visible(a, len - 1) : 0, keep = (int)a.keep_first;
  return Visible{lo, keep < lo ? keep : lo};
}

// The blocks of SIZE tokens with anything to see, numbered from 0: `kept` from the start of the sequence, then those from block
// `first` on, up to the one that holds token end - 1.
template <int SIZE>
struct VisibleBlocks {
  int first, kept;
  __device__ __forceinline__ VisibleBlocks(int lo, int keep_first) : first(lo / SIZE), kept((keep_first + SIZE - 1) / SIZE) {
    kept = kept < first ? kept : first;
  }
  __device__ __forceinline__ int count(int end) const { return kept + (end + SIZE - 1) / SIZE - first; }
  __device__ __forceinline__ int token(int block) const { return SIZE * (block < kept ? block : block - kept + first); }
};

// How a score comes about, in units of log 2.
enum ScoreKind {
  kSloped,         // scale and distance bias
  kCapped,         // scale and cap
  kCappedFixed     // the same with a cap so low that exponentials of scores need no reference: |score| <= kFixedCap
};
constexpr float kFixedCap = 64.f;      // e^64 times any sum of 2^20 values stays inside float32, e^-64 is a normal number with room for the low half

inline ScoreKind score_kind(const mops_hip_biased_attention& a) {
  return a.softcap > 0.f ? (a.softcap <= kFixedCap ? kCappedFixed : kCapped) : kSloped;
}

// cap tanh(dot scale / cap) = cap - 2 cap / (1 + e^(2 dot scale / cap)), times log2 e
struct CappedScore {
  float in, cap;
  __device__ __forceinline__ explicit CappedScore(const mops_hip_biased_attention& a)
      : in(a.softcap > 0.f ? 2.8853900817779268f * a.scale / a.softcap : 0.f), cap(1.4426950408889634f * a.softcap) {}
  __device__ __forceinline__ float operator()(float dot) const {
    return cap - 2.f * cap * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(in * dot));
  }
};

}  // namespace mops
