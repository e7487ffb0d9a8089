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
  kCappedFixed,    // the same with a cap so low that exponentials of scores need no reference: |score| <= kFixedCap
  kLogSloped,      // scale and a bias that grows with the logarithm of the distance
  kSigmoid         // no softmax: every key counts with the sigmoid of scale and a bias per head
};
constexpr bool needs_reference(ScoreKind kind) { return kind != kCappedFixed && kind != kSigmoid; }
constexpr float kFixedCap = 64.f;      // e^64 times any sum of 2^20 values stays inside float32, e^-64 is a normal number with room for the low half

inline ScoreKind score_kind(const mops_hip_biased_attention& a) {
  if (a.weight_bias) return kSigmoid;
  if (a.log_rate) return kLogSloped;
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

// A score in units of log 2 from the product of query and key and the distance between them.
template <ScoreKind KIND>
struct ScoreOf {
  CappedScore capped;
  float scale, slope, step, bias;
  __device__ __forceinline__ ScoreOf(const mops_hip_biased_attention& a, int h)
      : capped(a), scale(a.scale * 1.4426950408889634f),
        slope(KIND == kSloped && a.slopes ? a.slopes[h] * 1.4426950408889634f : (KIND == kLogSloped ? a.log_rate[h] : 0.f)),
        step(KIND == kLogSloped ? a.log_step[h] : 0.f), bias(KIND == kSigmoid ? a.weight_bias[h] * 1.4426950408889634f : 0.f) {}
  // behind: minus the distance
  __device__ __forceinline__ float operator()(float dot, float behind) const {
    if (KIND == kSloped) return dot * scale + slope * behind;
    if (KIND == kLogSloped) return dot * scale - slope * __builtin_amdgcn_logf(1.0f - step * behind);
    if (KIND == kSigmoid) return dot * scale + bias;
    return capped(dot);
  }
  // what a key counts: its exponential relative to a reference, or its sigmoid
  __device__ __forceinline__ float weight(float score, float reference) const {
    if (KIND == kSigmoid) return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-score));
    return __builtin_amdgcn_exp2f(score - reference);
  }
};

// The arguments with what zeros leave out.
inline mops_hip_biased_attention completed(const mops_hip_biased_attention& args) {
  mops_hip_biased_attention a = args;
  if (a.out_stride == 0) a.out_stride = a.heads * a.vdim;
  if (a.out_scale == 0.f) a.out_scale = 1.f;
  return a;
}

// What multiplies an output behind the division by the sum of weights: a gate per head, per element or none, and a constant.
template <typename T>
struct OutputGate {
  const T* g;
  float constant;
  bool each;
  __device__ __forceinline__ OutputGate(const mops_hip_biased_attention& a, int64_t row, int h)
      : g(a.gate ? (const T*)a.gate + row * a.gate_stride + (a.gate_each ? (int64_t)h * a.vdim : h) : nullptr), constant(a.out_scale),
        each(a.gate && a.gate_each) {
    if (g && !each) constant *= sigmoid_for<T>(to_f32(*g));
  }
  __device__ __forceinline__ float operator()(int v) const { return each ? constant * sigmoid_for<T>(to_f32(g[v])) : constant; }
};

}  // namespace mops
