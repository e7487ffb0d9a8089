/*
 * mops_hip.h — C ABI of libmops_hip.so: hand-written gfx950 (MI355X) kernels for the hot operators of
 * the `mops` operator library of nano_vllm_ninetoothed.
 *
 * Conventions for every launcher below
 *   - all pointers are DEVICE pointers unless stated; activations/caches/weights are bf16 (raw 16-bit
 *     words), metadata is int32 unless a flag says otherwise;
 *   - `stream` is a hipStream_t passed as void* (NULL = the default stream); the launch is asynchronous,
 *     nothing synchronises, nothing is allocated, nothing is freed;
 *   - return value: MOPS_HIP_OK (0) or a negative MOPS_HIP_E* status; on a negative status no kernel was
 *     launched.  Argument validation (null pointers, unsupported sizes, misalignment) happens on the host
 *     before launch, mirroring the reference's wrapper-side `assert`s.
 *
 * The reference has no native code: each entry point replaces the GPU kernel(s) behind one op name of
 * the reference's registry (mops/__init__.py:15-26), cited per function.
 */
#ifndef MOPS_HIP_H
#define MOPS_HIP_H

#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

#define MOPS_HIP_OK 0
#define MOPS_HIP_EINVAL (-1)       /* null pointer, negative size, inconsistent arguments            */
#define MOPS_HIP_EUNSUPPORTED (-2) /* shape the kernels are not written for (head_dim, block size…)  */
#define MOPS_HIP_EALIGN (-3)       /* pointer or stride breaks the 16-byte alignment the kernels need */
#define MOPS_HIP_EWORKSPACE (-4)   /* workspace missing or smaller than mops_hip_*_workspace_bytes    */
#define MOPS_HIP_ELAUNCH (-5)      /* a HIP call or launch reported an error (see mops_hip_last_hip_error) */
#define MOPS_HIP_ETOOLARGE (-6)    /* problem exceeds the fixed scratch of an allocation-free entry point */

/* ABI version of this header; bumped on any signature change. */
int mops_hip_abi_version(void);

/* Static, human-readable text for a status returned by any function here. */
const char* mops_hip_status_string(int status);

/* hipError_t (as int) of the last failed launch on this host thread, 0 if none. */
int mops_hip_last_hip_error(void);

/*
 * store_kvcache — slot_mapping scatter of freshly computed K and V rows into the paged cache.
 * Replaces: mops/triton/attention.py:7-38 (store_kvcache_kernel + wrapper), reached from
 * mops/torch/ops.py:62-65 and called at nanovllm/layers/attention.py:29.
 *
 *   for i in [0, n_tokens): s = slot_mapping[i]; if s == -1 skip;
 *       k_cache[s*row_elems : (s+1)*row_elems] = key[i*key_row_stride : +row_elems]   (same for V)
 *
 * key/value: rows of row_elems (= num_kv_heads*head_dim) contiguous bf16, row i at element offset
 * i*{key,value}_row_stride (strides in ELEMENTS, may exceed row_elems: V is a view into the qkv buffer).
 * k_cache/v_cache: contiguous [num_slots, row_elems].  Slots outside [0, num_slots) other than -1 are
 * skipped as well (the reference would write out of bounds).  Bit-exact copy.
 * Needs row_elems % 8 == 0, strides % 8 == 0 and 16-byte aligned base pointers.
 */
int mops_hip_store_kvcache(const void* key, int64_t key_row_stride,
                           const void* value, int64_t value_row_stride,
                           void* k_cache, void* v_cache,
                           const int32_t* slot_mapping,
                           int64_t n_tokens, int64_t row_elems, int64_t num_slots,
                           void* stream);

/*
 * embedding — row gather out[i, :] = weight[ids[i], :].
 * Replaces: mops/torch/ops.py:57-59 (F.embedding), mops/triton/embedding.py:6-50; called at
 * nanovllm/layers/embed_head.py:41.
 * ids: n_ids indices, int64 when ids_are_int64 != 0 else int32.  weight: [vocab, hidden] bf16 with row
 * stride weight_row_stride (elements).  out: contiguous [n_ids, hidden].  An id outside [0, vocab)
 * produces a zero row instead of a fault.  Bit-exact copy.  hidden % 8 == 0, stride % 8 == 0.
 */
int mops_hip_embedding(const void* ids, int ids_are_int64,
                       const void* weight, int64_t weight_row_stride,
                       void* out,
                       int64_t n_ids, int64_t vocab, int64_t hidden,
                       void* stream);

/*
 * rms_forward — y = bf16(bf16(x * rsqrt(mean(x^2) + eps)) * w), fp32 statistics, two bf16 roundings.
 * Replaces: mops/torch/ops.py:9-16, mops/triton/rms_forward.py:7-36; called at
 * nanovllm/layers/layernorm.py:21 (2-D hidden states and the 3-D strided q/k views of
 * nanovllm/models/qwen3.py:76-77).
 * x is addressed as x[(o*stride_outer + i*stride_inner) + 0..n) for o < rows_outer, i < rows_inner
 * (strides in elements); y is contiguous [rows_outer*rows_inner, n]; x is never written.
 * n % 8 == 0, n <= 16384, strides % 8 == 0.
 */
int mops_hip_rms_forward(const void* x, const void* weight, void* y,
                         int64_t rows_outer, int64_t rows_inner, int64_t n,
                         int64_t stride_outer, int64_t stride_inner,
                         float eps, void* stream);

/*
 * add_rms_forward — s = float(x) + float(residual); residual_out = bf16(s);
 *                   y = bf16(bf16(s * rsqrt(mean(s^2) + eps)) * w)   (statistics on the unrounded s).
 * Replaces: mops/torch/ops.py:18-30, mops/triton/add_rms_forward.py:7-39; called at
 * nanovllm/layers/layernorm.py:29.
 * x, residual: [rows, n] with row strides x_row_stride / residual_row_stride (elements); y and
 * residual_out contiguous [rows, n].  residual_out may alias residual (in-place convention of the
 * triton/ninetoothed backends) when residual is contiguous; y must not alias an input.
 */
int mops_hip_add_rms_forward(const void* x, int64_t x_row_stride,
                             const void* residual, int64_t residual_row_stride,
                             const void* weight,
                             void* y, void* residual_out,
                             int64_t rows, int64_t n,
                             float eps, void* stream);

/*
 * Paged decode attention (one query token per sequence against the block-table-addressed KV cache).
 * Replaces: flash_attn.flash_attn_with_kvcache as reached from mops/torch/ops.py:74-76 (semantics
 * spelled out in the commented torch version at mops/torch/ops.py:78-125) and the NineToothed kernel
 * mops/ninetoothed/attention.py:157-348; called at nanovllm/layers/attention.py:40-42.
 *
 *   out[b,h,:] = softmax_t( scale * q[b,h,:] . K[b,t,h/(hq/hkv),:] ) @ V[b,t,h/(hq/hkv),:],
 *   t in [0, cache_seqlens[b]),  token t at cache[block_table[b, t/block_size], t%block_size, kvhead, :]
 *
 * q: [batch, hq, 128] bf16, batch stride q_batch_stride elements (head stride 128).
 * k_cache/v_cache: contiguous [num_blocks, block_size, hkv, 128] bf16.
 * block_table: int32 [batch, *] with row stride block_table_row_stride, at least
 * max_blocks_per_seq columns; columns at or beyond ceil(cache_seqlens[b]/block_size) are never read
 * (they hold -1); an entry outside [0, num_blocks) inside the used range is treated as an empty block.
 * cache_seqlens[b] is clamped to [0, max_blocks_per_seq*block_size]; 0 gives a zero output row.
 * out: contiguous [batch, hq, 128] bf16.
 * workspace: device scratch of at least mops_hip_paged_decode_workspace_bytes(...) bytes, 256-byte
 * aligned, private to this call until it completes on `stream`.
 * Supported: head_dim 128, block_size a multiple of 32, hq/hkv <= 16, num_blocks >= 1.
 */
int64_t mops_hip_paged_decode_workspace_bytes(int64_t batch, int64_t hq, int64_t hkv,
                                              int64_t max_blocks_per_seq, int64_t block_size);

int mops_hip_attn_paged_decode_bf16(const void* q, int64_t q_batch_stride,
                                    const void* k_cache, const void* v_cache,
                                    const int32_t* cache_seqlens,
                                    const int32_t* block_table, int64_t block_table_row_stride,
                                    void* out,
                                    int64_t batch, int64_t hq, int64_t hkv, int64_t head_dim,
                                    int64_t block_size, int64_t num_blocks, int64_t max_blocks_per_seq,
                                    float softmax_scale,
                                    void* workspace, int64_t workspace_bytes,
                                    void* stream);

/*
 * The same with the planning step under the caller's control.  The plan (how the KV stream of the batch is
 * cut over the workgroups) depends only on cache_seqlens, the batch and head counts and the block size, not
 * on q or on the caches, so the layers of one decode step can share it: call the first layer with
 * MOPS_HIP_DECODE_PLAN_AND_ATTEND and the others, on the same stream with the same workspace and the same
 * metadata, with MOPS_HIP_DECODE_REUSE_PLAN.  "The same metadata" means the same CONTENTS: a plan records the batch and
 * the head geometry it was made for (a call whose batch or heads differ is refused: its output is zeros), but not the
 * lengths.  If cache_seqlens or block_table have been rewritten in place since the planning call (same pointers, new
 * values, as a serving loop's static buffers are), MOPS_HIP_DECODE_REUSE_PLAN follows the old split: rows come out
 * truncated or zero, and nothing reports it.  Plan again whenever the contents may have changed (once per decode
 * step).  No counterpart in the reference (its attention call is per layer, nanovllm/layers/attention.py:40-42).
 */
#define MOPS_HIP_DECODE_PLAN_AND_ATTEND 0
#define MOPS_HIP_DECODE_REUSE_PLAN 1
int mops_hip_attn_paged_decode_planned_bf16(const void* q, int64_t q_batch_stride,
                                            const void* k_cache, const void* v_cache,
                                            const int32_t* cache_seqlens,
                                            const int32_t* block_table, int64_t block_table_row_stride,
                                            void* out,
                                            int64_t batch, int64_t hq, int64_t hkv, int64_t head_dim,
                                            int64_t block_size, int64_t num_blocks, int64_t max_blocks_per_seq,
                                            float softmax_scale,
                                            void* workspace, int64_t workspace_bytes,
                                            int plan_mode, void* stream);

/*
 * Paged decode attention for callers that cannot allocate: code under HIP-graph capture, tight serving loops
 * that hold no workspace, harnesses that forbid hipMalloc.  No counterpart in the reference.  Arguments and
 * results are those of mops_hip_attn_paged_decode_bf16 (same kernels, bit-identical output) without the
 * workspace pair: the split-context partials live in a fixed device array inside the library, one copy of
 * MOPS_HIP_DECODE_NOALLOC_SCRATCH_BYTES per GPU, held until the process ends.  The call allocates and frees
 * nothing and does not synchronise.  A problem whose workspace (mops_hip_paged_decode_workspace_bytes) exceeds
 * that size returns MOPS_HIP_ETOOLARGE and launches nothing; both benchmark shapes fit (4.3 MB at 256
 * sequences x 16/8 heads, 8.5 MB at 512 x 32/8).  All calls on one GPU share that GPU's array: calls that
 * overlap in time on one GPU (different streams, or threads) race; calls on one stream are ordered and safe.
 * The first call on a GPU looks the array's device address up (hipGetSymbolAddress); make it outside capture.
 */
#define MOPS_HIP_DECODE_NOALLOC_SCRATCH_BYTES (16ll << 20)
int mops_hip_attn_paged_decode_noalloc_bf16(const void* q, int64_t q_batch_stride,
                                            const void* k_cache, const void* v_cache,
                                            const int32_t* cache_seqlens,
                                            const int32_t* block_table, int64_t block_table_row_stride,
                                            void* out,
                                            int64_t batch, int64_t hq, int64_t hkv, int64_t head_dim,
                                            int64_t block_size, int64_t num_blocks, int64_t max_blocks_per_seq,
                                            float softmax_scale, void* stream);

/*
 * Varlen (packed, THD) causal prefill attention with grouped-query heads, with or without a cached prefix.
 * Replaces: flash_attn.flash_attn_varlen_func as reached from mops/torch/ops.py:70-72 and the Triton
 * kernel mops/triton/attention.py:42-146; called at nanovllm/layers/attention.py:34-37 (with the paged
 * caches as k/v and block_table set when a prefix-cache hit occurred, attention.py:32-33).
 *
 *   for sequence s with query tokens [cu_q[s], cu_q[s+1]) and Lk = cu_k[s+1]-cu_k[s] keys (Lk >= Lq):
 *     out[i,h,:] = softmax_{j <= i + (Lk-Lq)}( scale * q[i,h,:] . K_s[j,h/(hq/hkv),:] ) @ V_s[j,h/(hq/hkv),:]
 *
 * q/out: [total_tokens, hq, 128] bf16, token strides in elements (multiples of 8), head stride 128.
 * block_table == NULL: k/v are packed [total_k_tokens, hkv, 128] with their own token strides (multiples of 8,
 *   at most 2^24 elements: MOPS_HIP_EUNSUPPORTED beyond) and key j of sequence s is row cu_k[s] + j;
 *   cu_seqlens_k may be NULL (then it equals cu_seqlens_q).
 * block_table != NULL: k/v are the contiguous paged caches [num_blocks, block_size, hkv, 128] and key j of
 *   sequence s is cache[block_table[s, j/block_size], j%block_size] (row stride block_table_row_stride,
 *   at least max_blocks_per_seq columns; entries beyond the sequence's keys are never read; an entry
 *   outside [0, num_blocks) inside the used range is treated as an empty block, i.e. its keys get no weight,
 *   the rule of the decode entry points; block_size must be a multiple of 64); k/v token strides are ignored.
 * cu_seqlens_*: int32 [batch+1], non-decreasing, starting at 0.  max_seqlen_q bounds every query length
 * and only sizes the launch.  Sequences of length 0 are allowed.  softmax_scale may be any finite value
 * (0: uniform weights over the visible keys).  The scale is applied to the fp32 scores in fp32; with
 * MOPS_HIP_PREFILL_PRESCALE=1 in the environment (read at the first call) Q is multiplied by
 * softmax_scale * log2(e) once and rounded back to bf16 instead: faster, less accurate for large scores.
 * Accuracy: max-abs 2e-2 and mean-abs 2e-3 against an fp32 reference for scores of the benchmark's size
 * (softmax_scale 128^-1/2 on N(0,1) data: outputs below 2, one bf16 ulp <= 0.0156).  The bound is one bf16 ulp of the
 * output, so it scales with the outputs: at softmax_scale 1 on the same data the outputs reach 4 (ulp 0.031) and the
 * tests allow max-abs 4e-2 there.
 * Launches with an even hq / hkv, up to 512 sequences and up to 65536 tokens per sequence whose keys are the sequences'
 * own tokens, and launches behind a cached prefix (cu_seqlens_k or block_table given) with at most 64 sequences, at
 * most 512 new tokens per sequence on average and, when paged, at most 768 block table entries
 * (batch * max_blocks_per_seq), keep two workgroups per CU resident and hand them work items through counters in a
 * device array inside the library (128 rows, one per launch, round robin, cleared by the launch): at most 128 such
 * launches may be in flight per device; a launch captured into a HIP graph keeps its row.  MOPS_HIP_PREFILL_FORM=rows
 * (read at the first call) keeps every launch on the one-workgroup-per-128-rows form the other inputs take.
 */
int mops_hip_attn_varlen_causal_bf16(const void* q, int64_t q_token_stride,
                                     const void* k, int64_t k_token_stride,
                                     const void* v, int64_t v_token_stride,
                                     void* out, int64_t out_token_stride,
                                     const int32_t* cu_seqlens_q, const int32_t* cu_seqlens_k,
                                     const int32_t* block_table, int64_t block_table_row_stride,
                                     int64_t block_size, int64_t num_blocks, int64_t max_blocks_per_seq,
                                     int64_t batch, int64_t total_tokens, int64_t total_k_tokens,
                                     int64_t max_seqlen_q,
                                     int64_t hq, int64_t hkv, int64_t head_dim,
                                     float softmax_scale,
                                     void* stream);

/*
 * siluAndMul — out = bf16( bf16(silu(x)) * y ), elementwise over [rows, n].
 * Replaces: mops/torch/ops.py:32-34 (F.silu(x) * y), mops/ninetoothed/activation.py:10-32; called at
 * nanovllm/layers/activation.py:16 with x, y the two halves of the gate_up projection (row strides in
 * elements; out contiguous [rows, n]).  n % 8 == 0, strides % 8 == 0.
 */
int mops_hip_silu_and_mul(const void* x, int64_t x_row_stride, const void* y, int64_t y_row_stride,
                          void* out, int64_t rows, int64_t n, void* stream);

/*
 * apply_rotary_emb — neox-style half-split rotation of x [tokens, heads, head_dim] bf16 by per-token
 * fp32 cos/sin rows of head_dim/2 values: y1 = x1*cos - x2*sin, y2 = x2*cos + x1*sin (fp32, products
 * rounded separately), out contiguous [tokens, heads, head_dim] bf16.
 * Replaces: mops/torch/ops.py:45-54, mops/ninetoothed/rotary_emb.py:10-65; called at
 * nanovllm/layers/rotary_embedding.py:35-36.  head_dim % 16 == 0.
 */
int mops_hip_apply_rotary_emb(const void* x, int64_t x_token_stride, int64_t x_head_stride,
                              const float* cos, int64_t cos_token_stride,
                              const float* sin, int64_t sin_token_stride,
                              void* out, int64_t tokens, int64_t heads, int64_t head_dim, void* stream);

/*
 * sampler_forward — out[r] = argmax(softmax(logits[r, :] / temperature[r])) for positive temperatures, i.e.
 * the index of the row's largest logit (first index on ties).  The temperatures do not change the result
 * and are not passed.  A row holding a NaN or +inf logit, or only -inf, gives 0: the library softmax turns such a row
 * into NaNs and its argmax of an all-NaN row is 0.  Not reproduced: temperatures <= 0 (the library expression yields
 * inf/NaN garbage) and logits so close to zero that they collide after the fp32 division and exponential
 * (|logit| / T below ~1e-5, where every candidate is equally tiny).  Replaces: mops/torch/ops.py:37-43 (greedy: the Gumbel line is commented out),
 * mops/ninetoothed/sampler_forward.py:9-94; called at nanovllm/layers/sampler.py:12.
 * logits: [rows, n] bf16 with row stride in elements (% 8 == 0); out: int64 [rows].
 */
int mops_hip_sampler_argmax(const void* logits, int64_t row_stride, int64_t* out, int64_t rows, int64_t n,
                            void* stream);

/*
 * An empty kernel on `stream`: what one launch costs on this device with nothing to do.  No counterpart in the
 * reference; it exists so that the durations of the small operators (norms, embedding at decode sizes) can be read
 * against a measured floor (bench.py --op launch_floor).
 */
int mops_hip_launch_floor(void* stream);

/*
 * qk_norm_rope_store — the four small steps between the qkv projection and the attention call of a Qwen3
 * layer as one launch: per-head RMSNorm of q and k, rotary embedding of both, scatter of k and v into the
 * paged cache.  Replaces the sequence nanovllm/models/qwen3.py:74-80 (q_norm, k_norm, rotary_emb) +
 * nanovllm/layers/attention.py:29-31 (store_kvcache), i.e. mops rms_forward x2, apply_rotary_emb x2 and
 * store_kvcache, and is bit-identical to running those (same roundings in the same order).
 * qkv: [tokens, (hq + 2*hkv) * 128] bf16, q heads first, then k, then v, token stride in elements (% 8 == 0);
 * q_weight, k_weight: [128] bf16; cos, sin: fp32 [tokens, 64] with token strides; slot_mapping: int32 [tokens],
 * -1 or out of range = skip the cache rows of that token; q_out: [tokens, hq, 128] bf16; k_out: [tokens, hkv, 128]
 * bf16 or NULL when the rotated keys are only needed in the cache (decode); caches: [num_slots, hkv, 128] bf16.
 * v is not copied out: the attention call reads it from qkv as a strided view.
 */
int mops_hip_qk_norm_rope_store(const void* qkv, int64_t qkv_token_stride, const void* q_weight,
                                const void* k_weight, const float* cos, int64_t cos_token_stride,
                                const float* sin, int64_t sin_token_stride,
                                const int32_t* slot_mapping, void* q_out, void* k_out, void* k_cache,
                                void* v_cache, int64_t tokens, int64_t hq, int64_t hkv, int64_t head_dim,
                                int64_t num_slots, float eps, void* stream);

/*
 * linear — y = x . W^T (+ bias), bf16 in and out, fp32 accumulation, as a library GEMM (hipBLASLt).
 * Replaces: mops/torch/ops.py:5-7 (F.linear), called from nanovllm/layers/linear.py:53,75,152 and
 * nanovllm/layers/embed_head.py:64.
 * x: [m, k] bf16, w: [n, k] bf16 (nn.Linear layout), y: [m, n] bf16, row strides in elements (% 8 == 0, as
 * are n and k); bias: [n] bf16 or NULL.  workspace: device scratch for solutions that split k (may be NULL
 * with workspace_bytes 0; solutions that need more than is given are not chosen).
 * The solution is the one pinned for (m, n, k) with mops_hip_linear_pin_solution if it supports the
 * problem; without a pin for m, the one pinned for the next larger row count with the same n and k; else the
 * first the library's heuristic returns.  Unlike the kernels above this entry point keeps
 * host-side state (a library handle per device, one descriptor per distinct shape).
 */
int mops_hip_linear_bf16(const void* x, int64_t x_row_stride, const void* w, int64_t w_row_stride,
                         const void* bias, void* y, int64_t y_row_stride,
                         int64_t m, int64_t n, int64_t k,
                         void* workspace, int64_t workspace_bytes, void* stream);

/* Pins the library solution `solution_index` (as returned by mops_hip_linear_tune on the same library
 * version) for problems with these m, n, k; a negative index removes the pin.  Host-only, no GPU work. */
int mops_hip_linear_pin_solution(int64_t m, int64_t n, int64_t k, int solution_index);

/*
 * Times every solution the library offers for (m, n, k) on `distinct_weights` different weight matrices used
 * in turn (so that none is served from cache, as in a decode step that walks through the layers), `rounds`
 * passes per measurement, and returns the index of the fastest, its time per GEMM in microseconds, and the
 * time of the heuristic's choice.  A set-up utility: it allocates and frees its own buffers, creates a
 * stream and synchronises; not for use on a hot path or under stream capture.  No counterpart in the
 * reference.
 */
int mops_hip_linear_tune(int64_t m, int64_t n, int64_t k, int64_t distinct_weights, int rounds,
                         void* workspace, int64_t workspace_bytes,
                         int* best_solution_index, float* best_us, float* heuristic_us);

/* ---------------------------------------------------------------------------------------------------------------------
 * Operators of models with recurrent layers, latent attention and a float32 residual stream.  No counterpart in the
 * reference.  They exist for two element types of activations, weights and caches, named by `dtype`; everything they
 * reduce, scale or carry from token to token is float32 either way.
 * Positions, state slots and sequence metadata are int32 on the device.
 * ------------------------------------------------------------------------------------------------------------------- */
#define MOPS_HIP_BF16 0
#define MOPS_HIP_F32 1

/* residual[i, :] = scale * table[ids[i], :] and act[i, :] = the same in `dtype`, rows act_stride apart (act may be NULL); an id outside
 * [0, vocab) gives zeros. */
int mops_hip_embed_residual(const int64_t* ids, const void* table, int64_t table_row_stride, int dtype, float scale,
                            float* residual, void* act, int64_t act_stride, int64_t n_ids, int64_t vocab, int64_t width, void* stream);

/*
 * residual [rows, n] float += y + shift, or = y + shift with `replace`; y (`dtype`, rows y_stride apart) and shift (float [n]) may be NULL.
 * out (`dtype`, rows out_stride apart, or NULL) = norm(residual) * w + b: RMS norms, or layer norms with `center`; w NULL: the residual.
 */
typedef struct {
  float* residual;
  const void* y;
  int64_t y_stride;
  const float* shift;
  const void *w, *b;
  void* out;
  int64_t out_stride, rows, n;
  float eps;
  int replace, center, dtype;
} mops_hip_add_norm_args;
int mops_hip_add_norm(const mops_hip_add_norm_args* a, void* stream);

/* residual += y / sqrt(mean(y^2) + eps) * (weight_offset + weight), rowwise and in place; act = the new residual in `dtype`. */
int mops_hip_norm_residual_add(float* residual, const void* y, int64_t y_row_stride, const void* weight, float weight_offset,
                               float eps, void* act, int dtype, int64_t rows, int64_t n, void* stream);

/*
 * residual = scale * table[id] + pairs[(token in front * mul_prev + id * mul_cur) mod buckets], and pairs[buckets] for a sequence's
 * first token; table [vocab, width], pairs [buckets + 1, width].  The token in front of a sequence's first token of the step is
 * before[state_slots[b]] (none where starts[b] == 0 or the slot is negative), which receives the sequence's last token.
 * token_seq and cu_seqlens (both or neither): packed portions; NULL: one token per sequence.
 */
typedef struct {
  const int64_t* ids;
  const void *table, *pairs;
  int64_t table_stride, pairs_stride, buckets, mul_prev, mul_cur;
  int32_t* before;
  int64_t num_slots;
  const int32_t *token_seq, *cu_seqlens, *starts, *state_slots;
  float* residual;
  int64_t tokens, vocab, width;
  float scale;
  int dtype;
} mops_hip_embed_pairs_args;
int mops_hip_embed_pairs(const mops_hip_embed_pairs_args* a, void* stream);

/*
 * Norms behind one sublayer and in front of the next: with y_r the sum of the rows r * parts .. r * parts + parts - 1 of y and of
 * row r of extra ([rows, n], or NULL),
 * residual_r += y_r / sqrt(mean(y_r^2) + eps) * w_out in place, out_r = residual_r / sqrt(mean(residual_r^2) + eps) * w_in.
 * center: both norms take the mean of their row off first.
 */
int mops_hip_add_norm_norm(float* residual, const void* y, int64_t y_row_stride, int64_t parts, const void* extra, const void* w_out,
                           const void* w_in, float eps, int center, void* out, int dtype, int64_t rows, int64_t n, void* stream);

/* out = (x - mean(x)) / sqrt(mean((x - mean(x))^2) + eps) * weight of float32 rows. */
int mops_hip_layer_norm_f32(const float* x, const void* weight, float eps, void* out, int dtype, int64_t rows, int64_t n, void* stream);

/* out = x / sqrt(mean(x^2) + eps) * (weight_offset + weight) of float32 rows. */
int mops_hip_rms_norm_f32(const float* x, const void* weight, float weight_offset, float eps, void* out, int dtype,
                          int64_t rows, int64_t n, void* stream);

/*
 * Rows of groups * group_size elements, every group divided by its own root mean square:
 *   gate_first == 0:  out = rms(y) * silu(gate) [* weight];  else  out = rms(y * silu(gate)) [* weight].   weight may be NULL.
 * plain_sigmoid: sigmoid(gate) in the place of silu(gate).  shared_weight: weight [group_size] for all groups.  Everything times scale.
 * out may be y itself when their strides agree.
 */
int mops_hip_gated_group_norm(const void* y, int64_t y_row_stride, const void* gate, int64_t gate_row_stride,
                              const void* weight, int shared_weight, float eps, int gate_first, int plain_sigmoid, float scale, void* out,
                              int64_t out_row_stride, int dtype, int64_t rows, int64_t groups, int64_t group_size, void* stream);

/* out = g * sigmoid(alpha * g) * (u + 1), g = min(gate, limit), u = clamp(up, -limit, limit). */
int mops_hip_clamped_glu(const void* gate, int64_t gate_row_stride, const void* up, int64_t up_row_stride, void* out,
                         int64_t out_row_stride, int dtype, int64_t rows, int64_t n, float alpha, float limit, void* stream);
/* out = gelu(gate) * up, gelu(z) = z (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3))) / 2. */
int mops_hip_gelu_glu(const void* gate, int64_t gate_row_stride, const void* up, int64_t up_row_stride, void* out,
                      int64_t out_row_stride, int dtype, int64_t rows, int64_t n, void* stream);
/* out = max(gate, 0) * up. */
int mops_hip_relu_glu(const void* gate, int64_t gate_row_stride, const void* up, int64_t up_row_stride, void* out,
                      int64_t out_row_stride, int dtype, int64_t rows, int64_t n, void* stream);

/*
 * A linear recurrence with one decay per head and token (see csrc/decayed_recurrence.hip):
 *   S_t = a_t S_(t-1) + k_t (s_t v_t)^T,   o_t = S_t^T q_t + skip v_t
 * q, k: [tokens, groups * d], v, out: [tokens, heads * vd] with token strides in elements; value head h uses q/k head
 * h / (heads / groups).  Exactly one of `decay` (float [heads]: constant), `dt` ([tokens, heads] in `dtype`, with
 * dt_bias and neg_a float [heads]: s = softplus(dt + dt_bias), a = exp(neg_a * s)) and `channel_decay` is given; skip may be NULL.
 * channel_decay: float [tokens, heads * d], natural logarithms of a decay per token, head and key channel, with a token stride
 * in elements; then groups == heads, no skip and no convolution, and with bonus u (float [heads * d])
 *   o_t = (S_(t-1) + diag(u) k_t v_t^T)^T q_t,   S_t = diag(a_t) S_(t-1) + k_t v_t^T
 * rot > 0 rotates dimensions i and i + rot/2 of q and k (i < rot/2) by row `position` of cos_sin [max_positions, rot]
 * (cosines, then sines); k is multiplied by k_scale afterwards.
 * cu_seqlens: int32 [batch + 1], or NULL when every sequence brings one token.  starts[b]: position of the first token of
 * the portion; 0 starts from a zero state whatever the slot holds.
 * state: float [num_slots, heads, vd, pitch], pitch = mops_hip_recurrence_state_pitch(d); state_slots[b] < 0: a padding
 * row, out is zeros and nothing is stored.
 * conv_weight != NULL (one token per sequence only): the short convolution of mops_hip_short_conv is applied to q, k and v
 * on the way in, channels q_channel.. k_channel.. v_channel.. of `channels`, and the ring receives the token.
 * d <= 512.
 */
typedef struct {
  const void *q, *k, *v;
  int64_t q_stride, k_stride, v_stride;
  void* out;
  int64_t out_stride;
  float* state;
  int64_t num_slots;
  const int32_t *state_slots, *cu_seqlens, *starts;
  const float *decay, *log_decay, *neg_a, *dt_bias, *skip, *cos_sin;
  const void* dt;
  int64_t dt_stride;
  int64_t batch, heads, groups, d, vd, rot, max_positions;
  const float *conv_weight, *conv_bias;
  void* conv_ring;
  int64_t taps, channels, q_channel, k_channel, v_channel;
  const float *channel_decay, *bonus;
  int64_t channel_decay_stride;
  float k_scale;
  int dtype;
  const void *input_gate, *forget_gate;
  int64_t gate_stride;
  const float *input_bias, *forget_bias;
  float* top;
  const float *log_keep, *input_scale, *least;
  float gate_cap;
} mops_hip_recurrence;
/*
 * Matrix memory (input_gate given, in the place of a decay): gates are `dtype` [tokens, heads] with rows gate_stride apart, biases float
 * [heads]; k_scale multiplies q; state [num_slots, heads, vd + copies, pitch] and top float [num_slots, heads, copies], copies = mops_hip_matrix_memory_copies.
 * The chunked form takes the gates from mops_hip_matrix_memory_gates instead: log_keep, input_scale and least, float [tokens, heads].
 */
int64_t mops_hip_matrix_memory_copies(int64_t vd);
int mops_hip_matrix_memory_gates(const mops_hip_recurrence* r, float* log_keep, float* input_scale, float* least, void* stream);
int64_t mops_hip_recurrence_state_pitch(int64_t d);
int mops_hip_decayed_recurrence(const mops_hip_recurrence* r, void* stream);

/*
 * The same for portions of many tokens, 64 tokens at a time on the matrix cores (csrc/decayed_chunks.hip).  bf16 only, d <= 256, no
 * convolution, cu_seqlens required; a constant decay is read from log_decay (natural logarithms, finite) instead of decay.
 * segments: int32 [num_segments][3] = (sequence, first token, one past the last); the segments of a sequence are consecutive,
 * in order, and cover it.  seg_state == NULL: one segment per sequence.  Otherwise seg_state: float [num_segments, heads,
 * vd, pitch], seg_decay: float [num_segments, heads] are scratch, and seq_segments: int32 [batch + 1] bounds each
 * sequence's segments.  mops_hip_decayed_chunks_workgroups: workgroups one segment gives, for the choice of their number.
 */
int64_t mops_hip_decayed_chunks_workgroups(int64_t heads, int64_t groups, int64_t vd);
int mops_hip_decayed_chunks(const mops_hip_recurrence* r, const int32_t* segments, int64_t num_segments,
                            const int32_t* seq_segments, float* seg_state, float* seg_decay, void* stream);

/*
 * The same for a decay per key channel (csrc/channel_chunks.hip): 16 tokens at a time, bf16, d <= 256, channel_decay and bonus
 * given, no rotation, k_scale 1; a decay below 2^-28 counts as 2^-28.  seg_decay: float [num_segments, heads, pitch].
 */
int64_t mops_hip_channel_chunks_workgroups(int64_t heads, int64_t vd);
int mops_hip_channel_chunks(const mops_hip_recurrence* r, const int32_t* segments, int64_t num_segments,
                            const int32_t* seq_segments, float* seg_state, float* seg_decay, void* stream);

/*
 * The gated delta rule (csrc/delta_rule.hip): S <- exp(log_decay) S, u = sigmoid(beta) (v - S^T k), S <- S + k u^T, o = S^T q, with q and k
 * divided by sqrt(sum of squares + unit_eps) per head and q multiplied by q_scale.  q, k: [tokens, groups * d], v, out: [tokens, heads *
 * vd], beta: [tokens, heads] in `dtype`, log_decay: float [tokens, heads * d], all with row strides in elements; state: float [num_slots,
 * heads, vd, pitch], pitch = mops_hip_recurrence_state_pitch(d).  Sequences, slots and the convolution (without a bias) as in
 * mops_hip_recurrence.  d <= 512.
 */
typedef struct {
  const void *q, *k, *v;
  int64_t q_stride, k_stride, v_stride;
  void* out;
  int64_t out_stride;
  float* state;
  int64_t num_slots;
  const int32_t *state_slots, *cu_seqlens, *starts;
  const float* log_decay;
  const void* beta;
  int64_t log_decay_stride, beta_stride;
  int64_t batch, heads, groups, d, vd;
  const float* conv_weight;
  void* conv_ring;
  int64_t taps, channels, q_channel, k_channel, v_channel;
  float q_scale, unit_eps;
  int dtype;
} mops_hip_delta;
int mops_hip_delta_rule(const mops_hip_delta* a, void* stream);

/*
 * The same for portions of many tokens, 16 tokens at a time on the matrix cores (csrc/delta_chunks.hip): bf16, d <= 256, cu_seqlens given,
 * no convolution; a decay below 2^-28 counts as 2^-28.  chunks: int32 [num_chunks][2] = (first token, tokens <= 16): every sequence cut
 * from its first token on, in order.  segments: int32 [num_segments][4] = (sequence, first token, one past the last, number of its first
 * chunk): runs of whole chunks that cover every sequence, in order; seq_segments: int32 [batch + 1] bounds each sequence's.  One segment
 * per sequence, or more where that leaves the chip idle (mops_hip_delta_chunks_workgroups: what one segment gives).  workspace: device
 * scratch of at least mops_hip_delta_chunks_workspace_bytes(...), private to the call until it completes.
 */
int64_t mops_hip_delta_chunks_workgroups(int64_t heads, int64_t vd);
int64_t mops_hip_delta_chunks_workspace_bytes(int64_t num_chunks, int64_t num_segments, int64_t batch, int64_t heads, int64_t d, int64_t vd);
int mops_hip_delta_chunks(const mops_hip_delta* a, const int32_t* chunks, int64_t num_chunks, const int32_t* segments, int64_t num_segments,
                          const int32_t* seq_segments, void* workspace, int64_t workspace_bytes, void* stream);

/*
 * out[t, c] = silu(bias[c] (bias may be NULL) + sum over lags l < taps of weight[taps-1-l, c] * x(position - l)[c]) for packed portions.
 * weight: float [taps, channels]; x of earlier portions comes from ring [num_slots, taps, channels] (`dtype`), row
 * position % taps; positions before 0 count as zeros.  token_seq: int32 [tokens], the sequence of each token.
 */
int mops_hip_short_conv(const void* x, int64_t x_row_stride, const float* weight, const float* bias, const void* ring,
                        int64_t num_slots, const int32_t* token_seq, const int32_t* cu_seqlens, const int32_t* starts,
                        const int32_t* state_slots, void* out, int dtype, int64_t tokens, int64_t channels, int64_t taps,
                        void* stream);
/* Files the last taps-1 inputs of every portion in the ring; launch it behind everything that still reads the ring. */
int mops_hip_short_conv_update(const void* x, int64_t x_row_stride, void* ring, int64_t num_slots, const int32_t* cu_seqlens,
                               const int32_t* starts, const int32_t* state_slots, int dtype, int64_t batch, int64_t channels,
                               int64_t taps, void* stream);

/*
 * Latent attention (see csrc/latent_attention.hip).  latent_prepare: down [tokens, q_rank + kv_rank + rot_dim] ->
 * q_latent [tokens, q_rank] = RMS norm * q_weight; cache row slot_mapping[t] of [num_slots, pitch] =
 * [RMS norm of the kv latent * kv_weight | key part rotated in pairs (2i, 2i+1) | zeros]; slot < 0: no cache row.
 */
int mops_hip_latent_prepare(const void* down, int64_t down_stride, const void* q_weight, const void* kv_weight, float eps,
                            const float* cos_sin, int64_t max_positions, const int32_t* positions, const int32_t* slot_mapping,
                            void* q_latent, void* cache, int64_t num_slots, int64_t pitch, int dtype, int64_t tokens,
                            int64_t q_rank, int64_t kv_rank, int64_t rot_dim, void* stream);

/* y[t, h, :] = w[h] x[t, h, :] with w [heads, n, k] contiguous; token and head strides in elements. */
int mops_hip_head_linear(const void* x, int64_t x_token_stride, int64_t x_head_stride, const void* w, void* y,
                         int64_t y_token_stride, int64_t y_head_stride, int dtype, int64_t tokens, int64_t heads, int64_t n,
                         int64_t k, void* stream);

/*
 * Query rows against the latent cache: row r sees the first context_lens[r] tokens of sequence row_seq[r] (row r itself when
 * row_seq is NULL), its own position being context_lens[r] - 1; 0 gives zeros.  q_latent [rows, heads, kv_rank] contiguous,
 * q_rot the rot_dim query values (not yet rotated) at token / head strides, out [rows, heads, kv_rank] contiguous.
 * cache: [num_blocks, block_size, pitch]; a block table entry outside [0, num_blocks) counts as an empty block.
 */
typedef struct {
  const void *q_latent, *q_rot;
  int64_t q_rot_token_stride, q_rot_head_stride;
  const void* cache;
  int64_t pitch;
  const float* cos_sin;
  int64_t max_positions;
  const int32_t *row_seq, *context_lens, *block_table;
  int64_t block_table_stride, block_size, num_blocks, max_blocks;
  void* out;
  int64_t rows, heads, kv_rank, rot_dim;
  float scale;
  int dtype;
} mops_hip_latent_rows;
int mops_hip_latent_attention_rows(const mops_hip_latent_rows* a, void* stream);

/*
 * The same on the matrix cores (csrc/latent_decode.hip): bf16, kv_rank <= 512, kv_rank + rot_dim <= 576, block_size a
 * multiple of 32, pitch a multiple of 8; MOPS_HIP_EUNSUPPORTED otherwise.  workspace: device scratch of at least
 * mops_hip_latent_decode_workspace_bytes(...), private to the call until it completes.
 */
int64_t mops_hip_latent_decode_workspace_bytes(int64_t rows, int64_t heads, int64_t kv_rank, int64_t rot_dim);
int mops_hip_latent_decode(const mops_hip_latent_rows* a, void* workspace, int64_t workspace_bytes, void* stream);

/*
 * Long portions (csrc/latent_prefill.hip), bf16.  latent_gather: row i of c [rows, c_pitch] and kr [rows, kr_pitch] = latent and
 * key part of token row_pos[i] of sequence row_seq[i] (zeros for row_pos < 0 and in the padding columns).
 * rotate_pairs: x [tokens, heads, rot], pairs (2i, 2i+1) rotated in place by row positions[t] of cos_sin.
 * latent_prefill: q [tokens, heads, dim + rot_dim] (rotated), k [rows, heads * dim], kr [rows, rot_dim], vt [heads * vdim, rows],
 * out [tokens, heads, vdim] contiguous; dim, rot_dim and all strides of the inputs are multiples of 8 (pad with zeros).
 * tiles: int32 [num_tiles][5] = (first query token, queries <= 128, position of the first query, first key row, keys of the
 * context); the key rows of a context start at a multiple of 64 and the rows up to the next multiple of 64 exist.
 * dim + rot_dim <= 256, vdim <= 256.
 */
int mops_hip_latent_gather(const void* cache, int64_t pitch, const int32_t* block_table, int64_t table_stride, int64_t block_size,
                           int64_t num_blocks, int64_t max_blocks, const int32_t* row_seq, const int32_t* row_pos, void* c,
                           int64_t c_pitch, void* kr, int64_t kr_pitch, int64_t rows, int64_t kv_rank, int64_t rot_dim,
                           void* stream);
int mops_hip_rotate_pairs(void* x, int64_t token_stride, int64_t head_stride, const int32_t* positions, const float* cos_sin,
                          int64_t max_positions, int64_t tokens, int64_t heads, int64_t rot, void* stream);
int mops_hip_latent_prefill(const void* q, int64_t q_token_stride, int64_t q_head_stride, const void* k, int64_t k_stride,
                            const void* kr, int64_t kr_stride, const void* vt, int64_t vt_stride, const int32_t* tiles,
                            int64_t num_tiles, void* out, int64_t heads, int64_t dim, int64_t rot_dim, int64_t vdim, float scale,
                            void* stream);

/*
 * Time mixing (csrc/token_mix.hip).  token_mix: out[p][t] = x[t] + (x[t-1] - x[t]) * mu[p], mu float [parts, width], out
 * [parts, tokens, width].  The row in front of a sequence's first token of the step is row state_slots[b] of before
 * [num_slots, width] (zeros where starts[b] == 0 or the slot is negative), which receives the sequence's last row.
 * token_seq and cu_seqlens (both or neither): packed portions; NULL: one token per sequence.
 * low_rank_decay: out[t, c] = -exp(sum over r of w2[c, r] tanh(z[t, r]) + w0[c]), float; rank <= 4096.  With rate (float
 * [channels / head_size], else NULL) out[t, c] = rate[c / head_size] * softplus(sum over r of w2[c, r] z[t, r] + w0[c]).
 */
int mops_hip_token_mix(const void* x, int64_t x_row_stride, const float* mu, int64_t parts, void* before, int64_t num_slots,
                       const int32_t* token_seq, const int32_t* cu_seqlens, const int32_t* starts, const int32_t* state_slots,
                       void* out, int dtype, int64_t tokens, int64_t width, void* stream);
int mops_hip_low_rank_decay(const void* z, int64_t z_row_stride, const void* w2, const float* w0, const float* rate, int64_t head_size,
                            float* out, int dtype, int64_t tokens, int64_t channels, int64_t rank, void* stream);

/* out = max(x, 0)^2. */
int mops_hip_squared_relu(const void* x, int64_t x_row_stride, void* out, int dtype, int64_t rows, int64_t n, void* stream);

/*
 * Attention with a linear distance bias (csrc/biased_attention.hip).  With dp and vp the sizes dim and vdim rounded up to
 * multiples of 8: q [rows, heads, dp], k_pages [num_slots or num_blocks * block_size, kv_heads, dp], v_pages [.., kv_heads, vp].
 * attention_prepare: qkv rows [heads * dim | kv_heads * dim | kv_heads * vdim]; q = RMS norm over all of its elements * q_weight *
 * q_factor[position] (q_factor: float [max_positions], or NULL), k = RMS norm over all of its elements * k_weight; k and v go to
 * row slot_mapping[t] of the pages (slot < 0: nowhere).  Padding is written as zeros.
 */
typedef struct {
  const void* qkv;
  int64_t qkv_stride;
  const void *q_weight, *k_weight;
  const float* q_factor;
  int64_t max_positions;
  const int32_t *positions, *slot_mapping;
  void *q, *k_pages, *v_pages;
  int64_t num_slots, tokens, heads, kv_heads, dim, vdim;
  float eps;
  int dtype;
} mops_hip_attention_prepare_args;
int mops_hip_attention_prepare(const mops_hip_attention_prepare_args* a, void* stream);

/*
 * rotary_prepare (csrc/rotary_prepare.hip): the same for rotated queries and keys.  q_weight, k_weight [dim] or NULL: an RMS norm over
 * every head of q or k.  Then the pairs (i, i + rot / 2) of a head's first `rot` elements turn by the angles of the token's position:
 * cos_sin float [max_positions, rot], cosines, then sines.  neighbours: the pairs are (2i, 2i + 1).  bias (`dtype`, as many elements as
 * q, k and v have together, or NULL) is added in front of all that.
 */
typedef struct {
  const void* qkv;
  int64_t qkv_stride;
  const void *q_weight, *k_weight;
  const float* cos_sin;
  int64_t max_positions, rot;
  const int32_t *positions, *slot_mapping;
  void *q, *k_pages, *v_pages;
  int64_t num_slots, tokens, heads, kv_heads, dim, vdim;
  float eps;
  int dtype;
  const void* bias;
  int64_t neighbours;
} mops_hip_rotary_prepare_args;
int mops_hip_rotary_prepare(const mops_hip_rotary_prepare_args* a, void* stream);

/*
 * Query row r (at position context_lens[r] - 1) sees the first context_lens[r] tokens of sequence row_seq[r] (row r itself when
 * row_seq is NULL); 0 gives zeros.  score = q . k * scale - slopes[h] * distance (slopes float [heads], or NULL), softmax,
 * out [rows, heads, vdim].  A block table entry outside [0, num_blocks) counts as an empty block.
 * Zeros in the fields behind dtype leave out what they describe:
 *   softcap     score = softcap * tanh(q . k * scale / softcap); not together with slopes
 *   window      position i sees the last `window` tokens up to itself
 *   chunk       position i sees the tokens of its chunk up to itself, chunks of `chunk` tokens from position 0 on; not with window
 *   keep_first  the first keep_first tokens stay visible
 *   sinks       float [heads]: exp(sinks[h]) is one more term of the softmax's denominator
 *   gate        `dtype` [rows, heads], or with gate_each [rows, heads * vdim], rows gate_stride apart: out is multiplied by its sigmoid
 *   log_rate    float [heads], with log_step [heads]: score = q . k * scale - log_rate[h] * ln(1 + log_step[h] * distance)
 *   weight_bias float [heads]: no softmax; a key counts with sigmoid(q . k * scale + weight_bias[h]).  Not with sinks
 * At most one of softcap, slopes, log_rate and weight_bias.  Rows of out are out_stride apart (0: contiguous) and
 * multiplied by out_scale (0: by one).
 * biased_attention_rows: the plain form; dim <= 2048, vdim <= 1024.
 */
typedef struct {
  const void *q, *k_pages, *v_pages;
  const float* slopes;
  const int32_t *row_seq, *context_lens, *block_table;
  int64_t block_table_stride, block_size, num_blocks, max_blocks;
  void* out;
  int64_t rows, heads, kv_heads, dim, vdim;
  float scale;
  int dtype;
  float softcap;
  int64_t window, chunk, keep_first;
  const float* sinks;
  const void* gate;
  int64_t gate_stride;
  const float *log_rate, *log_step, *weight_bias;
  int64_t gate_each, out_stride;
  float out_scale;
} mops_hip_biased_attention;
int mops_hip_biased_attention_rows(const mops_hip_biased_attention* a, void* stream);

/*
 * The same on the matrix cores: bf16, dim <= 256, vdim <= 256.
 * biased_decode (csrc/biased_decode.hip): single rows; block_size a multiple of 32.  workspace: device scratch of at least
 * mops_hip_biased_decode_workspace_bytes(...), private to the call until it completes.
 * biased_prefill (csrc/biased_prefill.hip): long portions.  q and out cover `rows` rows; tiles: int32 [num_tiles][5] = (first query
 * row, queries <= 128, position of the first query, block table row, tokens of the context); row_seq is not read and context_lens
 * only has to be there.  Writes the tiles' rows of out.
 */
int64_t mops_hip_biased_decode_workspace_bytes(int64_t rows, int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim);
int mops_hip_biased_decode(const mops_hip_biased_attention* a, void* workspace, int64_t workspace_bytes, void* stream);
int mops_hip_biased_prefill(const mops_hip_biased_attention* a, const int32_t* tiles, int64_t num_tiles, void* stream);

/*
 * Mixture of experts (csrc/moe.hip).  moe_route: logits = router [experts, width] h in float32; chosen, score [tokens * top] =
 * the experts with the largest logits and the sigmoids of these; rank [tokens * top] and counts [moe_route_workgroups(tokens),
 * experts] (aligned to 16 bytes) are scratch; rows [tokens * top] lists the choices (token * top + place) ordered by expert, tiles
 * [1 + 3 * moe_max_tiles] = number of blocks, then (expert, first row, rows) of each.  block_rows: 32, or 128 (bf16).
 * moe_gate_up: w [experts][2 * up_at][width], gate rows from 0, up rows from up_at on; y [tokens * top rows in the order of
 * `rows`], y = silu(score W_gate h) * (score W_up h).  moe_down: w [experts][width][depth], depth >= ff, the columns behind ff
 * zeros in w and finite in y; z [tokens * top] in the order of the choices.  experts <= 1024.
 * The weighted form, groups > 0: the experts are `groups` equal runs of neighbours; a choice score is sigmoid(logit) + correction[e]
 * (float [experts]), a group's score the sum of its two largest ones; the best `top` experts of the best `keep` groups are chosen, and
 * score = factor * sigmoid(logit) over the sum of the chosen ones' + 1e-20.  moe_down multiplies by it, and moe_gate_up does not.
 * unit 1: moe_gate_up gives g sigmoid(alpha g) (u + 1) with g = min(W_gate h, limit), u = W_up h between -limit and limit.
 * common_w: a unit that every token goes through, in the same launches (bf16, block_rows 32, unit 1; NULL: none).  moe_gate_up:
 * common_x [tokens, width], common_w gate rows from 0 and up rows from common_up_at on, [.., width], common_out [tokens, common_ff];
 * moe_down: common_x [tokens, common_ff], common_w [width, common_ff], common_out [tokens, width].
 */
typedef struct {
  int32_t *rows, *tiles;
  float* score;
  int64_t tokens, experts, top, width, ff, block_rows;
  int dtype;
  int unit;
  float limit, alpha;
  const float* correction;
  int64_t groups, keep;
  float factor, common_limit;
  const void *common_x, *common_w;
  void* common_out;
  int64_t common_x_stride, common_out_stride, common_ff, common_up_at;
} mops_hip_moe;
int64_t mops_hip_moe_max_tiles(int64_t tokens, int64_t experts, int64_t top, int64_t block_rows);
int64_t mops_hip_moe_route_workgroups(int64_t tokens);
int mops_hip_moe_route(const void* h, int64_t h_row_stride, const void* router, int32_t* chosen, int32_t* rank, int32_t* counts,
                       const mops_hip_moe* m, void* stream);
int mops_hip_moe_gate_up(const void* h, int64_t h_row_stride, const void* w, int64_t up_at, void* y, int64_t y_row_stride,
                         const mops_hip_moe* m, void* stream);
/* bf16: y[g, t] = w[g] x[g, t] with x [groups (+ 1), tokens, k], w [groups, n, k], y [groups, tokens, n], all contiguous.  w_last
 * [n_last <= n, k] (or NULL): weights of one more group of rows, y_last [tokens, n_last].  For batches of up to a few hundred tokens. */
int mops_hip_grouped_linear(const void* x, const void* w, void* y, const void* w_last, void* y_last, int64_t n_last, int64_t groups,
                            int64_t tokens, int64_t n, int64_t k, void* stream);
int mops_hip_moe_down(const void* y, int64_t y_row_stride, const void* w, int64_t depth, void* z, int64_t z_row_stride,
                      const mops_hip_moe* m, void* stream);

#ifdef __cplusplus
}
#endif
#endif /* MOPS_HIP_H */
