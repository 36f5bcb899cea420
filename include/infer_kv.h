/* infer_kv.h - C ABI of libinfer_kv.so: the paged KV-cache hot path on MI355X (gfx950).
 *
 * Three pieces, one library:
 *   1. KV append         - slot_mapping-driven scatter of new K/V rows into the paged caches.
 *   2. Paged decode attn - block_table-gathered GQA attention of one query token per sequence.
 *   3. Block pool        - host-side allocator of cache blocks with a prefix cache.
 *
 * Conventions for every device entry point:
 *   - all pointers are device pointers unless the name says "host"; they are borrowed for the
 *     duration of the call on `stream` (a hipStream_t passed as void*; NULL = default stream);
 *   - the call only enqueues work: it never synchronises, never allocates, never frees, and
 *     never throws; it is safe to record into a HIP graph;
 *   - return value: 0 on success, a negative INFER_KV_E* code for a rejected argument, or a
 *     positive hipError_t reported by the launch;
 *   - element type is bfloat16 (the only type the reference instantiates: src/kvcache.cc:305),
 *     strides are in ELEMENTS, metadata is int32.
 *
 * The reference has no FFI of its own for this path: the append is a Triton kernel and the
 * attention is the pip package flash_attn, both called from Python.  Each declaration below
 * cites the reference call it replaces (paths into the reference tree).
 */
#ifndef INFER_KV_H
#define INFER_KV_H

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

#define INFER_KV_OK            0
#define INFER_KV_EINVAL       -1   /* null pointer, non-positive size, unsupported shape        */
#define INFER_KV_EALIGN       -2   /* pointer or stride not aligned for the vector path         */
#define INFER_KV_EWORKSPACE   -3   /* workspace too small                                       */
#define INFER_KV_EUNSUPPORTED -4   /* head_dim / group size / block size outside what is built  */
#define INFER_KV_ESTATE       -5   /* block pool: the call violates an invariant the reference
                                      asserts (double allocate, out of blocks, ...); see
                                      infer_pool_last_error()                                   */
#define INFER_KV_EBUSY        -7   /* the library's own scratch array is still in use by work
                                      pending on another stream (infer_paged_decode_noalloc_bf16) */
/* element type of the entry points that take `elem` */
#define INFER_ELEM_BF16        0
#define INFER_ELEM_F32         1

#define INFER_KV_ENOTINIT     -6   /* first decode call on this device made while its stream is
                                      being captured: call infer_kv_init() before the capture    */

/* Library version, "major.minor". */
const char* infer_kv_version(void);

/* Human-readable text for a code returned by any entry point (negative codes: this library;
 * positive: hipGetErrorString). */
const char* infer_kv_strerror(int code);

/* One-time set-up for the CURRENT device (host only, no stream work): the decode kernels' LDS limit
 * (hipFuncSetAttribute), the compute-unit count and the address of the library's own scratch array
 * (hipGetSymbolAddress).  Every decode entry point does the same on its first call on a device, but
 * not while its stream is being captured (INFER_KV_ENOTINIT then): a caller that captures HIP graphs
 * calls this once per device beforehand.  Thread safe; later calls return at once. */
int infer_kv_init(void);

/* ------------------------------------------------------------------ 1. KV append
 * Replaces store_kvcache / store_kvcache_kernel (infer/ops/attention.py:16-45), called from
 * Attention.forward_offical_fa_impl (infer/ops/attention.py:108-109).
 *
 * For every row i in [0, n_rows): slot = slot_mapping[i]; if 0 <= slot < num_slots then
 *   k_cache[slot * dkv .. +dkv) = key[i * key_stride0 .. +dkv)   (same for value -> v_cache).
 * Rows whose slot is negative (padding) or >= num_slots are skipped; the reference has no such
 * guard (a -1 slot writes out of bounds there).  dkv = num_kv_heads * head_dim; the caches are
 * [num_slots, dkv] row-major (the reference asserts k_cache.stride(1) == dkv).  key/value rows
 * may be strided views of a fused qkv projection (row stride != dkv) but each row is contiguous.
 * Duplicate slots in one call race (last writer unspecified), as in the reference.
 * Requires dkv % 8 == 0 and 16-byte aligned rows (pointers and strides), else INFER_KV_EALIGN.
 */
int infer_kv_append_bf16(const void* key, int64_t key_stride0,
                         const void* value, int64_t value_stride0,
                         void* k_cache, void* v_cache,
                         const int32_t* slot_mapping,
                         int64_t n_rows, int64_t dkv, int64_t num_slots,
                         void* stream);

/* The dense per-sequence view that the getters of the reference's cache pool promise (Tensor<T>
 * get_key_cache / get_value_cache, include/kvcache.hpp:47-48: [len, heads, head_size] contiguous): tokens
 * 0 .. num_tokens-1 of ONE sequence gathered from the paged cache [num_blocks, block_size, dkv] through its
 * block-table row (device memory, ceil(num_tokens / block_size) entries, clamped into [0, num_blocks)) into
 * out [num_tokens, dkv].  The attention kernels never need it (they gather on the fly); it serves callers
 * that want a sequence's K or V as one tensor, and is the inverse of the append (bit-exact copy).
 * Requires dkv % 8 == 0 and 16-byte aligned pointers. */
int infer_kv_gather_bf16(const void* cache, const int32_t* block_table_row,
                         int64_t num_tokens, int64_t dkv, int64_t block_size, int64_t num_blocks,
                         void* out, void* stream);

/* ------------------------------------------------------------------ 1b. fused QK-norm + RoPE + KV append
 * Replaces, in one launch, the four steps in front of attention in QwenAttention.forward
 * (infer/models/Qwen3.py:113-131): q_norm and k_norm (RMSNorm.rms_forward, infer/ops/norm.py:63-73,
 * per head over head_dim with a [head_dim] bf16 weight), the in-place neox rotary embedding
 * (rotary_embedding_kernel, src/operators/rope/rope.cu:43-133; rot_dim == head_dim) and
 * store_kvcache (infer/ops/attention.py:16-45).
 *
 * q [n_rows, Hq, D] and k [n_rows, Hkv, D] (row strides in elements, heads contiguous) are
 * normalised and rotated; q is updated in place; the new k row goes to k_cache[slot] and, when
 * write_k_inplace != 0, also back into k; the v row is copied to v_cache[slot].  Rows whose slot is
 * negative or >= num_slots update q (and k in place) only.  positions are int64 and are clamped
 * into [0, max_position); cos_sin_cache is [max_position, D] bf16 = cos(D/2) | sin(D/2) per row.
 * Arithmetic rounds where the reference rounds (see the kernel source).  head_dim must be 128.
 */
int infer_kv_qk_norm_rope_append_bf16(void* q, int64_t q_stride0, void* k, int64_t k_stride0,
                                      const void* v, int64_t v_stride0,
                                      const int64_t* positions,
                                      const void* q_norm_weight, const void* k_norm_weight, float eps,
                                      const void* cos_sin_cache, int64_t max_position,
                                      void* k_cache, void* v_cache, const int32_t* slot_mapping,
                                      int64_t n_rows, int64_t num_q_heads, int64_t num_kv_heads,
                                      int64_t head_dim, int64_t num_slots,
                                      int write_k_inplace, void* stream);

/* ------------------------------------------------------------------ 2. paged decode attention
 * Replaces flash_attn_with_kvcache(q[B,1,Hq,D], k_cache, v_cache, cache_seqlens=context_lens,
 * block_table=block_tables, softmax_scale=scale, causal=True) at infer/ops/attention.py:118-120,
 * and is the body the stub src/operators/flashattn/flashattn_decode.cu:11-13 never got.
 *
 *   out[b, h, :] = softmax_t( scale * q[b, h, :] . K_b[t, h / G, :] ) V_b[t, h / G, :],
 *   t in [0, context_lens[b]),  G = num_q_heads / num_kv_heads,
 *   K_b[t] = k_cache[block_table[b, t / block_size], t % block_size]   (same for V).
 *
 * Rows with context_lens[b] <= 0 (graph padding) write zeros.  Table entries past
 * ceil(len / block_size) are never read; entries that are read are clamped into
 * [0, num_blocks) so a corrupt table cannot fault the GPU, and a length beyond what a table row can
 * address (table_cols * block_size) is cut to that, so a corrupt length cannot make the gather run
 * past its row.
 *
 * Layouts (strides in elements): q [B, Hq, D] with row stride q_stride0, heads contiguous;
 * out likewise with out_stride0; caches [num_blocks, block_size, Hkv, D] with block stride
 * cache_block_stride and token stride cache_token_stride (heads contiguous, D innermost);
 * block_table [B, table_cols] with row stride bt_stride0 >= table_cols; context_lens [B].
 *
 * The work is cut into equal shares of KV tokens regardless of sequence boundaries, one share per
 * wavefront.  Partial (max, sum, accumulator) results of one sequence that meet inside a workgroup are
 * folded there and go to `workspace` as one record; a second small kernel folds the records of a
 * sequence that reaches into neighbouring workgroups and writes the result.  Size the workspace with
 * infer_paged_decode_workspace_bytes() for the largest batch that will be passed; its contents need
 * no initialisation.  Calls that share a workspace must be ordered on one stream (the records of one
 * call are live until its merge kernel has run); calls on different streams need a workspace each.
 *
 * split_workgroups: span positions (workgroups per group of KV heads along the token axis) of this
 * call, 0 = choose from the device's compute-unit count (the tuned default), at most 1024.  The
 * library keeps no state between calls: two calls may use different counts, also concurrently.
 *
 * Built for head_dim == 128, 1 <= G <= 16, block_size % 32 == 0 (the reference requires a
 * multiple of 256: infer/config.py:21).
 */
size_t infer_paged_decode_workspace_bytes(int64_t max_batch, int64_t num_q_heads,
                                          int64_t num_kv_heads, int64_t head_dim);

int infer_paged_decode_bf16(const void* q, int64_t q_stride0,
                            const void* k_cache, const void* v_cache,
                            int64_t cache_block_stride, int64_t cache_token_stride,
                            void* out, int64_t out_stride0,
                            const int32_t* block_table, int64_t bt_stride0, int64_t table_cols,
                            const int32_t* context_lens,
                            int64_t batch, int64_t num_q_heads, int64_t num_kv_heads,
                            int64_t head_dim, int64_t block_size, int64_t num_blocks,
                            float scale, int64_t split_workgroups,
                            void* workspace, size_t workspace_bytes,
                            void* stream);

/* The two phases of infer_paged_decode_bf16 on their own: `split` streams the KV cache and leaves
 * partial results in the workspace, `merge` combines them into `out`.  Calling split then merge
 * on one stream is exactly infer_paged_decode_bf16.  They serve callers that want the partial results
 * themselves (a context-parallel split across devices would exchange exactly these records) and
 * profilers that time the bandwidth-bound phase alone.  The merge finds the records from the
 * workspace alone, so it does not need to know the split count. */
int infer_paged_decode_split_bf16(const void* q, int64_t q_stride0,
                                  const void* k_cache, const void* v_cache,
                                  int64_t cache_block_stride, int64_t cache_token_stride,
                                  const int32_t* block_table, int64_t bt_stride0, int64_t table_cols,
                                  const int32_t* context_lens,
                                  int64_t batch, int64_t num_q_heads, int64_t num_kv_heads,
                                  int64_t head_dim, int64_t block_size, int64_t num_blocks,
                                  float scale, int64_t split_workgroups,
                                  void* workspace, size_t workspace_bytes,
                                  void* stream);

int infer_paged_decode_merge_bf16(void* out, int64_t out_stride0,
                                  const int32_t* context_lens,
                                  int64_t batch, int64_t num_q_heads, int64_t num_kv_heads,
                                  int64_t head_dim,
                                  const void* workspace, size_t workspace_bytes,
                                  void* stream);

/* The decode call with the context length given as ONE host integer for the whole batch, the
 * `cache_seqlens: int` form of flash_attn_with_kvcache (the function called at
 * infer/ops/attention.py:118-120; the reference itself passes the per-sequence tensor, so this form is
 * NOT on the reference's call path).  Same result as infer_paged_decode_bf16 with
 * context_lens[b] == context_len for every b; context_len == 0 gives zeros.  Knowing the length, the
 * host can tell whether every sequence lies inside the spans of one workgroup (batch 64 x 512 ... 4096
 * tokens on 256 compute units do): the workgroups then write the result themselves and there is no
 * merge launch; other shapes run the two kernels of infer_paged_decode_bf16 without reading a lengths
 * array.  The workspace is the one of infer_paged_decode_bf16 (used by the second case). */
int infer_paged_decode_uniform_bf16(const void* q, int64_t q_stride0,
                                    const void* k_cache, const void* v_cache,
                                    int64_t cache_block_stride, int64_t cache_token_stride,
                                    void* out, int64_t out_stride0,
                                    const int32_t* block_table, int64_t bt_stride0, int64_t table_cols,
                                    int64_t context_len,
                                    int64_t batch, int64_t num_q_heads, int64_t num_kv_heads,
                                    int64_t head_dim, int64_t block_size, int64_t num_blocks,
                                    float scale,
                                    void* workspace, size_t workspace_bytes,
                                    void* stream);

/* infer_paged_decode_bf16 for callers that cannot allocate and have no workspace to bring: code under
 * HIP graph capture, tight serving loops, harnesses that forbid hipMalloc.  It has no counterpart in
 * the reference.  Same arguments, result and kernels as infer_paged_decode_bf16 with
 * split_workgroups = 0, but the split-KV records go to a fixed array in the library's device image
 * (16 MiB per GPU the library runs on, held by every process that loads the library until it ends,
 * whether or not this entry is called) instead of a workspace.  The call allocates nothing and frees
 * nothing.  Shapes whose records do not fit return INFER_KV_EWORKSPACE: the need is about
 * Hkv * (CUs * 4 / Hkv + batch) * 520 * G bytes, i.e. 3.2 MB at batch 64, Hq/Hkv = 32/8 and 4.5 MB at
 * batch 8, 64/8 on 256 compute units, against the INFER_KV_DECODE_NOALLOC_SCRATCH_BYTES of the array.
 * The array keeps the last call's contents and needs no clearing (every record that is read was
 * written by the same call).  All calls on one GPU share it: calls ordered on one stream are safe; a
 * call on another stream than the previous one is refused with INFER_KV_EBUSY while that stream still
 * has work pending (a cheap host-side check; calls racing on two host threads, and a capture that will
 * be replayed beside other users of the array, remain the caller's to order).  The address of the array is
 * resolved by infer_kv_init() or by the first decode call on the device outside stream capture. */
#define INFER_KV_DECODE_NOALLOC_SCRATCH_BYTES ((size_t)16 << 20)
int infer_paged_decode_noalloc_bf16(const void* q, int64_t q_stride0,
                                    const void* k_cache, const void* v_cache,
                                    int64_t cache_block_stride, int64_t cache_token_stride,
                                    void* out, int64_t out_stride0,
                                    const int32_t* block_table, int64_t bt_stride0, int64_t table_cols,
                                    const int32_t* context_lens,
                                    int64_t batch, int64_t num_q_heads, int64_t num_kv_heads,
                                    int64_t head_dim, int64_t block_size, int64_t num_blocks,
                                    float scale, void* stream);

/* ------------------------------------------------------------------ 2b. paged varlen prefill attention
 * Replaces flash_attn_varlen_func(Q, K, V, max_seqlen_q, cu_seqlens_q, max_seqlen_k, cu_seqlens_k,
 * softmax_scale, causal=True, block_table) at infer/ops/attention.py:110-116.
 *
 * Queries are packed: q [total_q, Hq, D] (row stride q_stride0), sequence s owns rows
 * [cu_seqlens_q[s], cu_seqlens_q[s+1]); out has the same layout.  Keys/values:
 *   block_table != NULL : k, v are the paged caches [num_blocks, block_size, Hkv, D] and sequence s
 *                         uses tokens [0, sk_s) of row s of the table, sk_s from cu_seqlens_k
 *                         (the reference's prefix-cache case, attention.py:111-112);
 *   block_table == NULL : k, v are packed rows [kv_rows, Hkv, D] indexed by cu_seqlens_k
 *                         (kv_token_stride is the row stride, kv_block_stride is ignored).
 * kv_rows = number of token rows addressable through k/v (packed: rows of the tensor; paged:
 * num_blocks * block_size); it only bounds reads.  causal != 0 applies the bottom-right aligned
 * mask (key j visible to query i of the sequence iff j <= i + (sk - sq)).  Queries of a sequence
 * with sk == 0 produce zeros, and so do the first sq - sk queries of a sequence with sq > sk (no key is
 * visible to them).  With a block table, table_cols is the number of entries per row
 * (bt_stride0 >= table_cols) and a key length beyond table_cols * block_size is cut to that.  scale
 * must be positive (INFER_KV_EINVAL otherwise).  Same shape limits as the decode entry points.  No
 * workspace.
 */
int infer_paged_prefill_bf16(const void* q, int64_t q_stride0,
                             const void* k, const void* v,
                             int64_t kv_block_stride, int64_t kv_token_stride, int64_t kv_rows,
                             void* out, int64_t out_stride0,
                             const int32_t* cu_seqlens_q, const int32_t* cu_seqlens_k,
                             const int32_t* block_table, int64_t bt_stride0, int64_t table_cols,
                             int64_t num_seqs, int64_t max_seqlen_q,
                             int64_t num_q_heads, int64_t num_kv_heads, int64_t head_dim,
                             int64_t block_size, int64_t num_blocks,
                             float scale, int causal, void* stream);

/* ------------------------------------------------------------------ 2c. the operators of a decode step around the path
 * What the engine runs between two attention calls of a captured decode step, so that the step is
 * HIP kernels of this library plus library GEMMs.
 *
 * infer_rms_norm_bf16 replaces RMSNorm.forward (infer/ops/norm.py:63-98; the torch path the engine
 * runs, rms_forward / add_rms_forward).  Without residual: out = bf16(x * rsqrt(mean(x^2) + eps)) *
 * weight.  With residual: s = float(x) + float(residual); residual <- bf16(s); out from the
 * unrounded s.  out may alias x.  Rows are [n_rows, hidden] bf16 with the given row strides
 * (elements); hidden % 8 == 0 and hidden <= 8192.
 */
int infer_rms_norm_bf16(const void* x, int64_t x_stride0, void* residual, int64_t residual_stride0,
                        const void* weight, void* out, int64_t out_stride0,
                        int64_t n_rows, int64_t hidden, float eps, void* stream);

/* Replaces silu_and_mul(result, input) (src/operators/silu/silu.cu:13-54; schema src/bindings.cpp:22):
 * out[r, j] = bf16(silu(x[r, j])) * x[r, d + j] for x [n_rows, 2 d] bf16, d % 8 == 0. */
int infer_silu_and_mul_bf16(void* out, int64_t out_stride0, const void* x, int64_t x_stride0,
                            int64_t n_rows, int64_t d, void* stream);

/* Replaces the host loop of ModelRunner.prepare_decode (infer/engine/model_runner.py:110-126) by
 * one launch on device-resident state.  seq_lens[b] = len(seq) including the token fed this step:
 *   context_lens[b] = len, positions[b] = len - 1 + position_offset,
 *   slot_mapping[b] = block_table[b, (len-1) / block_size] * block_size + (len-1) % block_size.
 * position_offset = 1 reproduces the reference (model_runner.py:117 feeds len(seq)); 0 gives the
 * zero-based position of its prefill branch (:84).  Rows with seq_lens[b] <= 0 (graph padding) get
 * slot -1, context length 0 and position 0, so they neither touch the cache nor attend. */
int infer_decode_metadata(const int32_t* seq_lens, const int32_t* block_table, int64_t bt_stride0,
                          int64_t batch, int64_t block_size, int64_t table_cols,
                          int64_t position_offset, int64_t* positions, int32_t* slot_mapping,
                          int32_t* context_lens, void* stream);

/* Replaces Linear.forward (infer/ops/MLP.py:103-149, F.linear; the op matmul(input, weight, output) of
 * src/bindings.cpp:7) at the batch sizes of a decode step, for weight matrices with few rows (o_proj,
 * down_proj): y[M, N] = x[M, K] . w[N, K]^T, bf16 in, float32 accumulate, bf16 out, M <= 128.  The
 * weights (row-major [N, K], contiguous) are streamed from HBM once; K is cut over workgroups and
 * float32 partial sums pass through `workspace` (infer_skinny_gemm_workspace_bytes says how much,
 * 0 if the shape needs no split).  K must be a multiple of 128 and N a multiple of 8; other shapes
 * return INFER_KV_EUNSUPPORTED and belong to the vendor GEMM. */
size_t infer_skinny_gemm_workspace_bytes(int64_t m, int64_t n, int64_t k);
int infer_skinny_gemm_bf16(const void* x, int64_t x_stride0, const void* w, void* y, int64_t y_stride0,
                           int64_t m, int64_t n, int64_t k, void* workspace, size_t workspace_bytes,
                           void* stream);
/* The same product without the final reduction, for a consumer that adds the partial sums itself
 * (infer_rms_norm_splitk_bf16): *splits_out > 1 means `workspace` now holds float32 partial sums
 * [splits][m][n] and y was not written; *splits_out == 1 means the shape needed no split and y holds
 * the bf16 result. */
int infer_skinny_gemm_partial_bf16(const void* x, int64_t x_stride0, const void* w, void* y, int64_t y_stride0,
                                   int64_t m, int64_t n, int64_t k, void* workspace, size_t workspace_bytes,
                                   int* splits_out, void* stream);
/* infer_rms_norm_bf16 whose input is still in pieces: x[r] = bf16(sum over s of partial[s][r]) with
 * partial[s][r] at partial + s * split_stride + r * partial_stride0 (float32 elements), added in
 * split order and rounded once - bit-identical to reducing first - then the same normalisation.
 * Fuses the reduction of a split-K o_proj / down_proj into the RMSNorm that follows it
 * (infer/models/Qwen3.py:226-236). */
int infer_rms_norm_splitk_bf16(const float* partial, int64_t splits, int64_t split_stride,
                               int64_t partial_stride0, void* residual, int64_t residual_stride0,
                               const void* weight, void* out, int64_t out_stride0,
                               int64_t n_rows, int64_t hidden, float eps, void* stream);

/* ------------------------------------------------------------------ operators of the hybrid models
 * Models that mix latent attention (one compressed cache row per token) with recurrent layers (one
 * fixed-size state per sequence) and keep the residual stream in float32.  No counterpart in the
 * reference.  `elem` is the element type of the activations, weights and cache rows behind the void
 * pointers (INFER_ELEM_*); norm weights, tables and recurrent state are float32. */

/* One pass over the rows of the float32 residual stream x[rows][width]:
 *   x = embed[tokens[row]] * embed_scale                    if tokens,
 *   x = x + y / sqrt(mean(y^2) + eps) * w_post              if y (element type) or partial (the float32
 *                                                           pieces of infer_skinny_gemm_partial_bf16),
 *   h = x / sqrt(mean(x^2) + eps) * w_pre                   if w_pre; h in the element type.
 * Token ids are clamped to the vocabulary. */
int infer_residual_norm(int elem, const int64_t* tokens, const void* embed, float embed_scale, int64_t vocab,
                        const void* y, int64_t y_stride, const float* partial, int64_t splits, int64_t split_stride,
                        int64_t partial_stride, const float* w_post, float* x, int64_t x_stride, const float* w_pre,
                        void* h, int64_t h_stride, int64_t n_rows, int64_t width, float eps, void* stream);

/* The same stream with the norm behind the sum (post-norm):
 *   x = embed[tokens[row]] * embed_scale                    if tokens,
 *   x = z / sqrt(mean(z^2) + eps) * w_post, z = alpha * x + y
 *                                                           if y or partial, as above,
 *   h = x, or x / sqrt(mean(x^2) + eps) * w_last if w_last  (always written). */
int infer_post_norm(int elem, const int64_t* tokens, const void* embed, float embed_scale, int64_t vocab,
                    const void* y, int64_t y_stride, const float* partial, int64_t splits, int64_t split_stride,
                    int64_t partial_stride, float alpha, const float* w_post, float* x, int64_t x_stride,
                    const float* w_last, void* h, int64_t h_stride, int64_t n_rows, int64_t width, float eps,
                    void* stream);

/* out[r, j] = gelu_tanh(x[r, j]) * x[r, d + j]. */
int infer_gelu_tanh_and_mul(int elem, void* out, int64_t out_stride, const void* x, int64_t x_stride,
                            int64_t n_rows, int64_t d, void* stream);
/* out[r, j] = silu(x[r, j]) * x[r, d + j], any d and strides (infer_silu_and_mul_bf16 rounds silu(x) to bf16
 * before the product, as the operator it replaces does; this one does not). */
int infer_silu_and_mul(int elem, void* out, int64_t out_stride, const void* x, int64_t x_stride,
                       int64_t n_rows, int64_t d, void* stream);
/* out[r][c] = g sigmoid(1.702 g) (u + 1) with g = min(x[r][c], limit), u = clamp(x[r][d + c], -limit, limit). */
int infer_clamped_gate_and_mul(int elem, void* out, int64_t out_stride, const void* x, int64_t x_stride, int64_t n_rows,
                               int64_t d, float limit, void* stream);

/* Front end of latent attention.  A token's projection row holds q (heads x [dim | rot]) at column 0 and
 * [latent: rank | rotated key part: rot] at column kv_off.  The latent is RMS-normed (c_norm), the first
 * rot_dims of every rotated part turn by the token's position (interleaved pairs; table[pos] = cos, sin per
 * pair), and the cache row [c | 0 .. rank_pad | rotated part | 0 .. row] is stored at slots[t] (negative:
 * skipped).  Rows below qx_rows get their rotated queries in qx[t][head][rank_pad .. row), zero padded, the
 * others in place. */
int infer_latent_front(int elem, void* proj, int64_t proj_stride, int64_t heads, int64_t dim, int64_t rot,
                       int64_t rot_dims, int64_t kv_off, int64_t rank, const float* c_norm, float eps,
                       const float* table, int64_t max_pos, const int64_t* positions, const int32_t* slots,
                       void* cache, int64_t rank_pad, int64_t row, int64_t num_slots, void* qx, int64_t qx_rows,
                       int64_t n, void* stream);

/* out[m][h][n] = sum_k x[m][h][k] w[h][n][k] (* sigmoid(gate[m][h]) if gate).  w rows are padded with zeros
 * to w_row elements (a multiple of 32) and every head to a multiple of 16 rows. */
int infer_head_matmul(int elem, const void* x, int64_t x_row, int64_t x_head, const void* w, int64_t w_head,
                      int64_t w_row, void* out, int64_t out_row, int64_t out_head, const void* gate, int64_t gate_row,
                      int64_t m, int64_t heads, int64_t n, int64_t k, void* stream);

/* Attention of query rows over paged latent rows.  qx[rows][heads][row] is dotted with the first ctx[r] cached
 * rows of the sequence in block-table row row_seq[r] (row_seq NULL: r), softmax of scale * score, and the
 * first rank_pad elements of the cached rows are summed: out[rows][heads][rank_pad].  `splits` is the number
 * of parts the keys are cut into (infer_latent_attention_splits gives a good one; the workspace holds
 * rows * splits * heads * (rank_pad + 2) floats if it is above 1). */
int64_t infer_latent_attention_splits(int elem, int64_t rows, int64_t heads, int64_t row, int64_t rank_pad,
                                      int64_t block_size, int64_t max_keys);
int infer_latent_attention(int elem, const void* qx, const void* cache, int64_t row, int64_t rank_pad,
                           const int32_t* block_table, int64_t bt_stride, int64_t table_cols, int64_t block_size,
                           int64_t num_blocks, const int32_t* row_seq, const int32_t* ctx, int64_t rows, int64_t heads,
                           float scale, int64_t splits, void* out, float* workspace, int64_t workspace_floats,
                           void* stream);

/* Cached rows (bf16) of whole sequences as dense rows: sequence s, in block-table row seqs[s], goes to rows
 * cu_k[s] .. cu_k[s + 1) of out[.][row]. */
int infer_latent_gather(const void* cache, int64_t row, int64_t block_size, int64_t num_blocks,
                        const int32_t* block_table, int64_t bt_stride, int64_t table_cols, const int32_t* seqs,
                        const int32_t* cu_k, int64_t num_seqs, int64_t max_keys, void* out, void* stream);

/* Causal varlen attention over dense keys [plain part per head | rotated part shared by all heads] and values
 * per head (bf16), output gated by sigmoid(gate[token][head]).  cu_q / cu_k: first token row / key row of each
 * sequence; query i sees keys 0 .. i + (sk - sq). */
int infer_latent_prefill_supported(int64_t dim, int64_t rot, int64_t vdim);
int infer_latent_prefill(const void* q, int64_t q_stride, const void* kp, int64_t kp_stride, const void* kr,
                         int64_t kr_stride, const void* v, int64_t v_stride, const void* gate, int64_t gate_stride,
                         void* out, int64_t out_stride, const int32_t* cu_q, const int32_t* cu_k, int64_t num_seqs,
                         int64_t max_seqlen_q, int64_t heads, int64_t dim, int64_t rot, int64_t vdim, float scale,
                         void* stream);

/* Grouped attention with separate keys and values: heads / kv_heads consecutive query heads share a key/value head.
 * Pages are [blocks][kv_heads][block_size][vdim_pad + dim_pad], a row holding the value, zeros, the key, zeros; both
 * parts are padded to 32 elements.
 *
 * infer_grouped_front: a token's projection row holds q (heads x dim) at column 0, k (kv_heads x dim) at k_off and v
 * (kv_heads x vdim) at v_off.  bias (per column, NULL: none) is added to all three; q and k are divided by the root
 * mean square of the WHOLE projection and multiplied by q_norm / k_norm (NULL: no norm); the first rot_dims entries of
 * every head turn by the token's position (interleaved pairs; table[pos] = cos, sin per pair); keys and values are
 * stored at slots[t] (negative: skipped).  kv_heads = 0: only q, the keys are another layer's.  Rows below qx_rows get
 * their q in qx[t][head][dim_pad], zero padded, the others in place.
 *
 * infer_grouped_attention: query rows against pages, as infer_latent_attention.  sink (NULL: none) is a score per head
 * that enters the softmax denominator and is not scaled; gate (NULL: none) multiplies a head's output by
 * sigmoid(gate[row][head]).  out[row][heads * vdim].
 *
 * infer_grouped_gather: as infer_latent_gather, out[.][kv_heads][row].
 * infer_grouped_prefill: as infer_latent_prefill over dense keys and values (bf16); head h reads key head
 * h / (heads / kv_heads), at k + that * k_head. */
int infer_grouped_front(int elem, void* proj, int64_t proj_stride, int64_t heads, int64_t kv_heads, int64_t dim,
                        int64_t vdim, int64_t k_off, int64_t v_off, const float* bias, const float* q_norm,
                        const float* k_norm, float eps, const float* table, int64_t rot_dims, int64_t max_pos,
                        const int64_t* positions, const int32_t* slots, void* cache, int64_t block_size,
                        int64_t dim_pad, int64_t vdim_pad, int64_t num_slots, void* qx, int64_t qx_rows, int64_t n,
                        void* stream);
int64_t infer_grouped_attention_splits(int elem, int64_t rows, int64_t heads, int64_t kv_heads, int64_t dim_pad,
                                       int64_t vdim_pad, int64_t block_size, int64_t max_keys);
int infer_grouped_attention(int elem, const void* qx, const void* cache, int64_t dim_pad, int64_t vdim_pad,
                            const int32_t* block_table, int64_t bt_stride, int64_t table_cols, int64_t block_size,
                            int64_t num_blocks, const int32_t* row_seq, const int32_t* ctx, int64_t rows,
                            int64_t heads, int64_t kv_heads, float scale, const float* sink, const void* gate,
                            int64_t gate_stride, int64_t splits, void* out, int64_t out_stride, int64_t vdim,
                            float* workspace, int64_t workspace_floats, void* stream);
int infer_grouped_gather(const void* cache, int64_t row, int64_t kv_heads, int64_t block_size, int64_t num_blocks,
                         const int32_t* block_table, int64_t bt_stride, int64_t table_cols, const int32_t* seqs,
                         const int32_t* cu_k, int64_t num_seqs, int64_t max_keys, void* out, void* stream);
int infer_grouped_prefill_supported(int64_t dim, int64_t vdim);
int infer_grouped_prefill(const void* q, int64_t q_stride, const void* k, int64_t k_stride, int64_t k_head, const void* v,
                          int64_t v_stride, int64_t v_head, const float* sink, const void* gate, int64_t gate_stride,
                          void* out, int64_t out_stride, const int32_t* cu_q, const int32_t* cu_k, int64_t num_seqs,
                          int64_t max_seqlen_q, int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim, float scale,
                          void* stream);

/* Pre-norm decoders with a learned scale behind every sublayer.
 *
 * infer_pre_norm, per row of the float32 stream x:  x <- x + y * scale [+ first] [+ step];  h <- rms(x) * w.
 * y is the sum of: the tensor y or the `splits` unreduced pieces of a split-K product; and for k < top, weights[row][k] times
 * row places[row][k] of `experts` (-1: the row itself of h_in).  scale, first and step may be NULL (1, 0, 0); first is
 * [row][width].  With `tokens` the sum is the embedding instead: embed[token] plus, with `bigram`, row
 * (prev * mul_prev + token * mul_cur) mod buckets of it (prev < 0: row `buckets`); first is then written (before step).
 * infer_softcap: out = cap * tanh(scale * x / cap), float32 [rows][cols]. */
int infer_pre_norm(int elem, const int64_t* tokens, const void* embed, int64_t vocab, const int64_t* prev,
                   const void* bigram, int64_t buckets, int64_t mul_prev, int64_t mul_cur, const void* y,
                   int64_t y_stride, const float* partial, int64_t splits, int64_t split_stride,
                   int64_t partial_stride, const void* experts, const int32_t* places, const float* weights,
                   int64_t top, int64_t num_places, const void* h_in, int64_t h_in_stride, const float* scale,
                   float* first, const float* step, float* x, int64_t x_stride, const float* w, void* h,
                   int64_t h_stride, int64_t n_rows, int64_t width, float eps, void* stream);
int infer_softcap(int elem, const void* x, int64_t x_stride, float* out, int64_t n_rows, int64_t cols, float cap,
                  float scale, void* stream);

/* Masked attention: pages [blocks][kv_heads][block_size][vdim_pad + key_pad], a row holding the value, zeros, the keys of
 * all maps one behind the other, zeros; both parts are padded to 32 elements.  maps = 2: a head has two queries and two keys
 * (head by head, map by map in the projections) beside one value.
 *
 * infer_head_front: projections q, k, v of a token at columns q_off, k_off, v_off; biases per column (NULL: none); RMS norm
 * per head (and map) with a weight [dim] (NULL: no norm); entry i < rot_dims / 2 turns with entry i + rot_dims / 2 by the token's
 * position; keys and values are stored at slots[t] (negative: skipped).  Rows below qx_rows get their q in
 * qx[t][head][map][key_pad] (zero where the other map's key stands), the others in place.
 *
 * infer_masked_attention: query rows against pages, as infer_grouped_attention.  mask_kind 0: all keys in front; 1: those of the
 * same chunk of mask_size tokens, counted from the sequence's start; 2: the last mask_size, itself among them.  biased: a score
 * loses 2^(-8 (h + 1) / heads) per token of distance.  The result is multiplied by out_scale.  maps = 2: the result is
 * rms(o1 - lambda o2) (eps) * out_scale, and the workspace always holds rows * splits * heads * 2 * (vdim_pad + 2) floats;
 * neither sink nor bias then.  Splits as infer_grouped_attention_splits for heads * maps heads and key_pad.
 * infer_masked_gather: as infer_grouped_gather, without the keys in front of what the first query of a portion sees.
 * infer_masked_prefill: as infer_grouped_prefill, gate optional; q [tokens][head][map][dim], k [keys][kv_head][map][dim]. */
int infer_head_front(int elem, void* proj, int64_t proj_stride, int64_t heads, int64_t kv_heads, int64_t maps,
                     int64_t dim, int64_t vdim, int64_t q_off, int64_t k_off, int64_t v_off, const float* bias,
                     const float* q_norm, const float* k_norm, float eps, const float* table, int64_t rot_dims,
                     int64_t max_pos, const int64_t* positions, const int32_t* slots, void* cache,
                     int64_t block_size, int64_t key_pad, int64_t vdim_pad, int64_t num_slots, void* qx,
                     int64_t qx_rows, int64_t n, void* stream);
int infer_masked_attention(int elem, const void* qx, const void* cache, int64_t key_pad, int64_t vdim_pad,
                           const int32_t* block_table, int64_t bt_stride, int64_t table_cols, int64_t block_size,
                           int64_t num_blocks, const int32_t* row_seq, const int32_t* ctx, int64_t rows,
                           int64_t heads, int64_t kv_heads, int64_t maps, float scale, int mask_kind,
                           int64_t mask_size, int biased, const float* sink, const void* gate, int64_t gate_stride,
                           float out_scale, float lambda, float eps, int64_t splits, void* out, int64_t out_stride,
                           int64_t vdim, float* workspace, int64_t workspace_floats, void* stream);
int infer_masked_gather(const void* cache, int64_t row, int64_t kv_heads, int64_t block_size, int64_t num_blocks,
                        const int32_t* block_table, int64_t bt_stride, int64_t table_cols, const int32_t* seqs,
                        const int32_t* cu_q, const int32_t* cu_k, int64_t num_seqs, int64_t max_keys, int mask_kind,
                        int64_t mask_size, void* out, void* stream);
int infer_masked_prefill_supported(int64_t maps, int64_t dim, int64_t vdim);
int infer_masked_prefill(const void* q, int64_t q_stride, const void* k, int64_t k_stride, int64_t k_head,
                         const void* v, int64_t v_stride, int64_t v_head, const float* sink, const void* gate,
                         int64_t gate_stride, void* out, int64_t out_stride, const int32_t* cu_q,
                         const int32_t* cu_k, int64_t num_seqs, int64_t max_seqlen_q, int64_t heads,
                         int64_t kv_heads, int64_t maps, int64_t dim, int64_t vdim, float scale, int mask_kind,
                         int64_t mask_size, int biased, float out_scale, float lambda, float eps, void* stream);

/* Float32 residual stream of a pre-norm decoder whose norm is a squashing function, norm(x) = tanh(alpha x) * w + b.  infer_tanh_norm:
 * x <- x + y + bias (y a tensor or split-K pieces as in infer_residual_norm, bias [width] or NULL), h <- norm(x).  With `tokens`
 * x <- the norm (in_alpha, in_w, in_b) of embed[token] * embed_scale instead.
 * infer_xielu: out = act(x + bias), act(z) = p z^2 + z / 2 for z > 0, q (e^z - 1 - z) + z / 2 otherwise. */
int infer_tanh_norm(int elem, const int64_t* tokens, const void* embed, int64_t vocab, float embed_scale, float in_alpha,
                    const float* in_w, const float* in_b, const void* y, int64_t y_stride, const float* partial,
                    int64_t splits, int64_t split_stride, int64_t partial_stride, const float* bias, float* x,
                    int64_t x_stride, float alpha, const float* w, const float* b, void* h, int64_t h_stride,
                    int64_t n_rows, int64_t width, void* stream);
int infer_xielu(int elem, const void* x, int64_t x_stride, const float* bias, float p, float q, void* out,
                int64_t out_stride, int64_t n_rows, int64_t cols, void* stream);

/* Talking-heads attention: softmax weights (one added to every denominator) of all heads are mixed by talk [heads][heads] before they
 * meet the values, w'_h = sum_g talk[h][g] w_g.  Pages of tiles of 32 tokens: keys [blocks][kv_heads][tile][key_pad / 8][token][8], values
 * [blocks][kv_heads][tile][vdim_pad / 16][token / 8][16][8 tokens]; both sizes are padded with zeros to 32 elements, block_size is a
 * multiple of 32.
 *
 * infer_unit_head_front: as infer_head_front for these pages; q, k and (norm_values) v of every head are divided by their root mean
 * square (eps), q is multiplied by 1 + temp_coef ln(floor((position + 1) / temp_every) + 1) (temp_every 0: by one).
 * infer_talking_attention: query rows qx [rows][heads][key_pad] against the first ctx[r] keys of the sequence in block-table row
 * row_seq[r] (NULL: r); ctx is at most max_keys.  out [rows][heads * vdim], multiplied by out_scale.  Between its kernels the scores
 * are in the workspace (infer_talking_attention_workspace_floats).
 * infer_talking_prefill: whole portions, bf16 (infer_talking_prefill_supported): q [tokens][head][dim], rows cu_q[s] .. cu_q[s + 1] are
 * the last tokens of the sequence in block-table row seqs[s], which has cu_k[s + 1] - cu_k[s] (at most
 * max_keys) keys; no score exceeds max_score (infinity: no bound is known); workspace: infer_talking_prefill_workspace_floats. */
int infer_unit_head_front(int elem, void* proj, int64_t proj_stride, int64_t heads, int64_t kv_heads, int64_t dim,
                          int64_t vdim, int64_t q_off, int64_t k_off, int64_t v_off, float eps, int norm_values,
                          float temp_coef, double temp_every, const int64_t* positions, const int32_t* slots, void* keys,
                          void* values, int64_t block_size, int64_t key_pad, int64_t vdim_pad, int64_t num_slots,
                          void* qx, int64_t qx_rows, int64_t n, void* stream);
int64_t infer_talking_attention_splits(int elem, int64_t rows, int64_t heads, int64_t kv_heads, int64_t key_pad,
                                       int64_t vdim_pad, int64_t block_size, int64_t max_keys);
int64_t infer_talking_attention_workspace_floats(int64_t rows, int64_t heads, int64_t vdim_pad, int64_t splits,
                                                 int64_t max_keys);
int infer_talking_attention(int elem, const void* qx, const void* keys, const void* values, int64_t key_pad,
                            int64_t vdim_pad, const int32_t* block_table, int64_t bt_stride, int64_t table_cols,
                            int64_t block_size, int64_t num_blocks, const int32_t* row_seq, const int32_t* ctx,
                            int64_t rows, int64_t heads, int64_t kv_heads, float scale, const void* talk, float out_scale,
                            int64_t splits, int64_t max_keys, void* out, int64_t out_stride, int64_t vdim,
                            float* workspace, int64_t workspace_floats, void* stream);
int infer_talking_prefill_supported(int64_t heads, int64_t dim, int64_t vdim);
int64_t infer_talking_prefill_workspace_floats(int64_t heads, int64_t vdim, int64_t num_seqs, int64_t tokens,
                                               int64_t max_seqlen_q, int64_t max_keys);
int infer_talking_prefill(const void* q, int64_t q_stride, const void* keys, const void* values, int64_t key_pad,
                          int64_t vdim_pad, const int32_t* block_table, int64_t bt_stride, int64_t table_cols,
                          int64_t block_size, int64_t num_blocks, const int32_t* seqs, const int32_t* cu_q,
                          const int32_t* cu_k, int64_t num_seqs, int64_t tokens, int64_t max_seqlen_q, int64_t max_keys,
                          int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim, float scale, const void* talk,
                          float out_scale, float max_score, void* out, int64_t out_stride, float* workspace, int64_t workspace_floats,
                          void* stream);

/* Selective state space: S <- e^{a dt} S + dt B x^T, y = S^T C + D x per head, dt = softplus(. + dt_bias), a = -e^{a_log}; x, B and C
 * behind a causal convolution per channel and silu, heads / groups consecutive heads share B and C; behind it
 * rms(y silu(z)) * norm over norm_parts equal parts of a row.  A projection row holds z [heads * vdim] at z_off, x, B
 * [groups * state_n] and C one behind the other at x_off, dt [heads] at dt_off.  conv [channels][taps], the last column for the
 * current token.  ring [slots][taps][channels] (position mod taps), state [slots][heads][state_n][vdim] float32.
 * Rows below decode_rows advance slots[r] by one token (negative: padding); the others belong to spans (first row, tokens,
 * slot, first position; max_span is the longest) and ring_slot[row] = (slot, rows of the span that follow).  xbc holds
 * (n - decode_rows) * channels elements, y n * heads * vdim. */
int64_t infer_state_space_workspace_floats(int elem, int64_t heads, int64_t vdim, int64_t state_n, int64_t num_spans,
                                           int64_t max_span);
int infer_state_space(int elem, const void* proj, int64_t proj_stride, int64_t z_off, int64_t x_off, int64_t dt_off,
                      int64_t heads, int64_t vdim, int64_t state_n, int64_t groups, int64_t taps, const float* conv,
                      const float* conv_bias, const float* dt_bias, const float* a_log, const float* d,
                      const float* norm, int64_t norm_parts, float eps, void* ring, float* state, int64_t num_slots,
                      const int32_t* slots, const int64_t* positions, int64_t decode_rows, const int32_t* spans,
                      int64_t num_spans, int64_t max_span, const int32_t* ring_slot, int64_t n, void* xbc, void* y,
                      float* workspace, int64_t workspace_floats, void* out, int64_t out_stride, void* stream);

/* Mixture of experts.  Router logits in float32, softmax over all experts + identity entries, choice scores = softmax +
 * correction (NULL: 0); of `groups` equal groups of neighbours the `keep` with the largest choice scores are open, of their
 * entries the `top` largest are chosen, with the softmax value times scale as weight.  Chosen experts (not identities) get a
 * row ("place") each: act = silu(gate) * up, out[place] = down act.  gate_up [experts][2 ff][width], down
 * [experts][width][ff_pad] (zero behind ff), act [places][ff_pad].  counts [experts] is zero before and after.  weights and places
 * (-1: identity) are [n][top]; ids, ranks, row_token, row_expert n * top, offsets experts + 1, tiles 2 * max_tiles integers.
 * infer_moe_layout: out = {places, tiles, rows per tile} for n tokens. */
int infer_moe_layout(int elem, int64_t n, int64_t width, int64_t ff_pad, int64_t experts, int64_t top, int64_t* out);
int infer_moe(int elem, const void* h, int64_t h_stride, const void* router, const float* correction, int64_t n,
              int64_t width, int64_t experts, int64_t identity, int64_t top, int64_t groups, int64_t keep,
              float scale, const void* gate_up, const void* down, int64_t ff, int64_t ff_pad, int32_t* counts,
              int32_t* ids, float* weights, int32_t* ranks, int32_t* places, int32_t* row_token, int32_t* row_expert,
              int32_t* offsets, int32_t* tiles, int64_t max_tiles, void* act, void* out, int64_t max_places,
              void* stream);

/* Linear attention with a constant decay d per head: S = d S + k v^T, o = scale * S^T q, S[dim][vdim] float32.  A
 * token's projection row holds q, k (heads x dim), v and the gate logits (heads x vdim) at q_off, k_off, v_off and
 * g_off.  silu: q, k and v go through silu; rot_dims > 0: the first rot_dims entries of every head of q and k turn by
 * the token's position, entry i with entry i + rot_dims / 2 (table[pos] = cos, sin per pair).  decay[3][heads] = d
 * rounded to float, d minus that, log2(d).  o is divided by its root mean square over the head (norm_per_head) or over
 * all heads, multiplied by norm[heads * vdim] (NULL: ones) and by sigmoid or silu of the gate.
 * Rows below decode_rows are single tokens with the state of slots[row] at positions[row] (a negative slot is padding:
 * zeros come out); the others belong to spans[.][4] = first row, tokens, slot, first position, two tokens or more.
 * state[slots][heads][rows][columns] (infer_decay_layout: [0] rows, [1] columns); a sequence at position 0 starts from
 * zero whatever it holds.  max_span: tokens of the longest span (a longer one is not computed whole); the workspace
 * holds infer_decay_workspace_floats floats. */
int infer_decay_layout(int64_t dim, int64_t vdim, int64_t* out2);
int64_t infer_decay_workspace_floats(int elem, int64_t heads, int64_t dim, int64_t vdim, int64_t rot_dims,
                                     int64_t num_spans, int64_t max_span);
int infer_decay_attention(int elem, const void* proj, int64_t proj_stride, int64_t q_off, int64_t k_off, int64_t v_off,
                          int64_t g_off, int64_t heads, int64_t dim, int64_t vdim, const float* decay, int silu,
                          const float* table, int64_t rot_dims, int64_t max_pos, float scale, const float* norm,
                          int norm_per_head, int gate_silu, float eps, float* state, int64_t num_slots,
                          const int32_t* slots, const int64_t* positions, int64_t decode_rows, const int32_t* spans,
                          int64_t num_spans, int64_t max_span, int64_t rows, float* workspace,
                          int64_t workspace_floats, void* out, int64_t out_stride, void* stream);

/* Gated delta rule with a decay per key channel.  A token's projection row holds the inputs of the short
 * convolution, q and k (kv_heads x dim each) and v (heads x vdim), from column 0 and the write-strength
 * logits (heads) at column beta_off; decay[row][heads * dim] and gate[row][heads * vdim] are the outputs of
 * the low-rank projections before softplus and sigmoid.  conv is [channels][taps], the last tap meeting the
 * current token.  ring[slots][taps][channels] and state[slots][heads][state rows][state columns] are the
 * sequence's state (infer_delta_layout: [0] state rows, [1] state columns, [2] floats of a chunk record,
 * [3] tokens per chunk); a sequence at position 0 starts from zero whatever they hold.
 *
 * infer_delta_step: one token per row; rows with a negative slot are padding (zeros come out).
 * infer_delta_chunks: prompt portions, rows row0 .. row0 + rows - 1.  portions[.][4] = first chunk, chunks, slot,
 * first position; chunks[.][6] = first row, tokens, first position, first position of the portion, slot, 0;
 * ring_slot[row][2] (indexed by batch row) = the slot, and how many rows of the portion follow.
 * records: num_chunks * heads * [2] floats; o: (row0 + rows) * heads * [1] floats. */
int infer_delta_layout(int64_t dim, int64_t vdim, int64_t* out4);
int infer_delta_step(int elem, const void* proj, int64_t proj_stride, int64_t beta_off, const void* decay,
                     int64_t decay_stride, const void* gate, int64_t gate_stride, const float* conv, const float* a_log,
                     const float* dt_bias, const float* norm, void* ring, float* state, int64_t num_slots, int64_t heads,
                     int64_t kv_heads, int64_t dim, int64_t vdim, int64_t taps, float eps, const int32_t* slots,
                     const int64_t* positions, void* out, int64_t out_stride, int64_t rows, void* stream);
int infer_delta_chunks(int elem, const void* proj, int64_t proj_stride, int64_t beta_off, const void* decay,
                       int64_t decay_stride, const void* gate, int64_t gate_stride, const float* conv, const float* a_log,
                       const float* dt_bias, const float* norm, void* ring, float* state, int64_t num_slots, int64_t heads,
                       int64_t kv_heads, int64_t dim, int64_t vdim, int64_t taps, float eps, const int32_t* portions,
                       int64_t num_portions, const int32_t* chunks, int64_t num_chunks, float* records, float* o,
                       const int32_t* ring_slot, const int64_t* positions, void* out, int64_t out_stride, int64_t row0,
                       int64_t rows, void* stream);

/* ------------------------------------------------------------------ 3. block pool (host only)
 * C view of infer::BlockPool (include/infer_kv/block_pool.hpp), the native counterpart of the
 * reference's Python BlockManager (infer/engine/block_mannager.py:44-133), which is the block
 * pool the reference engine runs (its C++ include/kvcache.hpp / src/kvcache.cc is never
 * compiled).  Token ids are int64, block ids int32.  Functions that the reference guards with
 * `assert` return INFER_KV_ESTATE and leave a message in infer_pool_last_error() (thread local).
 */
typedef struct infer_pool infer_pool;

infer_pool* infer_pool_create(int32_t num_blocks, int32_t block_size);   /* BlockManager.__init__ :46-52 */
void infer_pool_destroy(infer_pool* pool);
const char* infer_pool_last_error(void);
int32_t infer_pool_num_free(const infer_pool* pool);
int32_t infer_pool_num_used(const infer_pool* pool);

/* can_allocate :76-77 -> 1 / 0. */
int infer_pool_can_allocate(const infer_pool* pool, int64_t num_tokens);

/* allocate :79-103.  Writes ceil(num_tokens / block_size) block ids to table_out and returns the
 * number of tokens already present in the cache (a multiple of block_size), or a negative code. */
int64_t infer_pool_allocate(infer_pool* pool, const int64_t* token_ids, int64_t num_tokens,
                            int32_t* table_out, int64_t table_capacity);

/* deallocate :105-112 (references dropped in reverse table order). */
int infer_pool_deallocate(infer_pool* pool, const int32_t* table, int64_t num_blocks);

/* can_append :114-115 -> 1 / 0. */
int infer_pool_can_append(const infer_pool* pool, int64_t seq_len);

/* may_append :117-133, called after the sequence grew to seq_len tokens.  May append one block id
 * to `table` (capacity must allow num_blocks + 1 then).  Returns the new number of blocks. */
int64_t infer_pool_may_append(infer_pool* pool, const int64_t* token_ids, int64_t seq_len,
                              int32_t* table, int64_t num_blocks, int64_t table_capacity);
/* The same step given only the block_size tokens of the block that seq_len just filled (read only
 * when seq_len % block_size == 0, may be NULL otherwise), so a per-token caller does not have to
 * hand over the whole sequence. */
int64_t infer_pool_may_append_block(infer_pool* pool, const int64_t* last_block_tokens, int64_t seq_len,
                                    int32_t* table, int64_t num_blocks, int64_t table_capacity);

/* Takes `count` blocks from the front of the free list without hashing anything (sequences whose cache no
 * other sequence can share: part of their history is recurrent state).  All or nothing:
 * INFER_KV_ESTATE if fewer are free.  They go back through infer_pool_deallocate. */
int infer_pool_acquire(infer_pool* pool, int64_t count, int32_t* ids_out);

/* compute_hash :54-60: xxh64(seed 0) over [prefix hash as 8 LE bytes, if has_prefix] ++ int64 LE ids. */
uint64_t infer_pool_hash(const int64_t* token_ids, int64_t n, int has_prefix, uint64_t prefix_hash);

/* XXH64 itself (the reference gets it from the un-vendored pip package `xxhash`). */
uint64_t infer_xxh64(const void* data, size_t len, uint64_t seed);

/* Introspection. */
int32_t infer_pool_ref_count(const infer_pool* pool, int32_t block_id);
int infer_pool_block_hash(const infer_pool* pool, int32_t block_id, uint64_t* hash_out);  /* 1 if sealed */
int64_t infer_pool_free_ids(const infer_pool* pool, int32_t* out, int64_t capacity);      /* FIFO order */

#ifdef __cplusplus
}
#endif
#endif /* INFER_KV_H */
