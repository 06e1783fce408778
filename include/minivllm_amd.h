/*
 * minivllm_amd.h -- C ABI of libminivllm_amd.so (gfx950 / MI355X).
 *
 * The reference (Wenyueh/MinivLLM) is pure Python + Triton and has no FFI;
 * each entry point below replaces the Triton launch inside one of the
 * reference's Python operators and is what a ctypes binding of that operator
 * calls.  The reference location of the operator is cited per function.
 *
 * Conventions
 *   - every pointer is a DEVICE pointer unless stated otherwise;
 *   - `stream` is a hipStream_t passed as void* (NULL = the null stream);
 *   - return value: 0 ok, <0 invalid argument / unsupported shape
 *     (see mvllm_status_string), >0 a hipError_t from the launch;
 *   - the library never allocates, frees or synchronises; outputs and
 *     workspaces are caller-owned; launches have static grids derived from the
 *     host arguments only, so every call is legal under hipGraph capture;
 *   - tensors are dense row-major ("contiguous") in the stated shape.
 */
#ifndef MINIVLLM_AMD_H_
#define MINIVLLM_AMD_H_

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

/* element type of q/k/v/out and of a non-quantised KV cache */
enum mvllm_dtype {
  MVLLM_F32 = 0,
  MVLLM_BF16 = 1,
  MVLLM_F16 = 2,
};

/* negative status codes */
enum mvllm_status {
  MVLLM_OK = 0,
  MVLLM_ERR_NULL_POINTER = -1,
  MVLLM_ERR_BAD_DTYPE = -2,
  MVLLM_ERR_BAD_SHAPE = -3,      /* a size is <= 0 where it must be positive, or not divisible as required */
  MVLLM_ERR_UNSUPPORTED = -4,    /* shape valid but no kernel is built for it */
  MVLLM_ERR_WORKSPACE = -5,      /* workspace missing or smaller than *_workspace_bytes() */
  MVLLM_ERR_MISALIGNED = -6,     /* pointer not aligned to 16 bytes */
};

/* ABI version: major*1000 + minor. */
int mvllm_version(void);

/* Static, human-readable text for a status returned by this library
 * (negative codes only; positive codes are hipError_t). HOST pointer. */
const char* mvllm_status_string(int status);

/*
 * store_kvcache -- src/myvllm/layers/attention.py:67-108 (kernel :7-64).
 * For every token t with slot = slot_mapping[t]:
 *     slot == -1 (or outside [0, num_slots))  -> nothing is written
 *     else k_cache_flat[slot, :, :] = key[t, :, :], same for value,
 * where *_cache_flat is the [num_slots = num_blocks*block_size, Hkv, D] view of
 * the [num_blocks, block_size, Hkv, D] cache.  key/value: [T, Hkv, D], same
 * dtype as the caches (a bit-exact copy).  slot_mapping: int64 [T].
 */
int mvllm_store_kvcache(const void* key, const void* value,
                        void* k_cache, void* v_cache,
                        const int64_t* slot_mapping,
                        int64_t num_tokens, int64_t num_slots,
                        int num_kv_heads, int head_dim,
                        int dtype, void* stream);

/*
 * INT8 variant of store_kvcache (no counterpart in the reference; it serves
 * the same call site, attention.py:510, when the cache is int8).
 * Per (token, kv head): amax = max|x| in fp32, scale = amax / 127 (IEEE fp32
 * divide), code = clamp(rint(x / scale), -127, 127) (round half to even);
 * amax == 0 -> scale 0, codes 0.  Codes go to int8 caches [num_slots, Hkv, D],
 * scales to fp32 [num_slots, Hkv].  `dtype` is the dtype of key/value.
 */
int mvllm_store_kvcache_int8(const void* key, const void* value,
                             int8_t* k_cache, int8_t* v_cache,
                             float* k_scale, float* v_scale,
                             const int64_t* slot_mapping,
                             int64_t num_tokens, int64_t num_slots,
                             int num_kv_heads, int head_dim,
                             int dtype, void* stream);

/*
 * Bytes of fp32 split-K workspace mvllm_paged_decode{,_int8} need for these
 * static sizes (0 if the shape needs none).  Pure host arithmetic.
 */
size_t mvllm_paged_decode_workspace_bytes(int batch, int num_heads, int head_dim,
                                          int max_num_blocks, int block_size);

/*
 * How mvllm_paged_decode{,_int8} split these static sizes (no counterpart in the reference, whose Triton kernel
 * walks a whole context in one program, attention.py:283-415).  Pure host arithmetic:
 *   *part_tokens      tokens of a partition; partition p of a sequence covers tokens [p, p+1) * part_tokens
 *   *num_parts        partitions per sequence (1: no workspace is touched and no merge kernel is launched)
 *   *waves_per_head   1: a workgroup holds up to 4 kv heads, one wave each, and every wave walks its partition;
 *                     >1: small-batch form, a workgroup is that many waves on one kv head that share the
 *                     partition's 16-token tiles and merge in LDS; 0: the generic kernel (head_dim other than
 *                     128 or 64 (bf16 / fp16 caches: also every other multiple of 8 from 32 to 120, and 256),
 *                     a block_size that is neither a multiple of 16 nor, for 16-bit and fp32 caches with head_dim 128 or
 *                     64, one of 1, 2, 4, 8; or fp32 queries over an INT8 cache).  A kv head with more than 16 query
 *                     heads is served in slices of 16, each of which streams its keys and values again.
 * Returns MVLLM_OK or MVLLM_ERR_BAD_SHAPE / MVLLM_ERR_BAD_DTYPE.
 */
int mvllm_paged_decode_plan(int batch, int num_heads, int num_kv_heads, int head_dim,
                            int max_num_blocks, int block_size, int dtype, int int8_cache,
                            int* part_tokens, int* num_parts, int* waves_per_head);

/*
 * paged_attention_decode -- src/myvllm/layers/attention.py:418-473 (kernel :283-415).
 * out[b,h,:] = softmax_t( scale * q[b,h,:] . K[b,t,g(h),:] ) V[b,t,g(h),:],
 * t in [0, context_lens[b]), g(h) = h / (Hq/Hkv); token t of sequence b lives at
 * cache[block_tables[b, t / block_size], t % block_size, g, :].
 * Tokens whose table index is >= max_num_blocks, or whose entry is < 0 or
 * >= num_blocks, contribute nothing; context_len <= 0 gives a row of zeros.
 *   out, q        [batch, Hq, D]  `dtype`
 *   k/v_cache     [num_blocks, block_size, Hkv, D]  `dtype`
 *   block_tables  int32 [batch, max_num_blocks]
 *   context_lens  int64 [batch] if ctx_is_i64 else int32 [batch]
 *   workspace     >= mvllm_paged_decode_workspace_bytes(...) bytes, 16-byte aligned
 */
int mvllm_paged_decode(void* out, const void* q,
                       const void* k_cache, const void* v_cache,
                       const int32_t* block_tables, int max_num_blocks,
                       const void* context_lens, int ctx_is_i64,
                       int batch, int num_heads, int num_kv_heads, int head_dim,
                       int block_size, int64_t num_blocks, float scale, int dtype,
                       void* workspace, size_t workspace_bytes, void* stream);

/*
 * INT8-cache variant of paged decode (no counterpart in the reference).
 * K/V rows are dequantised in-kernel as code * scale in fp32.
 *   k/v_cache  int8 [num_blocks, block_size, Hkv, D]
 *   k/v_scale  fp32 [num_blocks, block_size, Hkv]
 *   `dtype` is the dtype of q and out.
 */
int mvllm_paged_decode_int8(void* out, const void* q,
                            const int8_t* k_cache, const int8_t* v_cache,
                            const float* k_scale, const float* v_scale,
                            const int32_t* block_tables, int max_num_blocks,
                            const void* context_lens, int ctx_is_i64,
                            int batch, int num_heads, int num_kv_heads, int head_dim,
                            int block_size, int64_t num_blocks, float scale, int dtype,
                            void* workspace, size_t workspace_bytes, void* stream);

/*
 * mvllm_paged_decode for callers that cannot allocate device memory (code under hipGraph capture, tight serving
 * loops, harnesses that forbid hipMalloc).  No counterpart in the reference.  Same arguments and results as
 * mvllm_paged_decode without the workspace: the split-K partials go to a static device array inside the library
 * (MVLLM_PAGED_DECODE_NOALLOC_MAX_BYTES per GPU, held until the process ends).  Shapes for which
 * mvllm_paged_decode_workspace_bytes() exceeds that size return MVLLM_ERR_WORKSPACE.  The call allocates and frees
 * nothing; the first call on a device looks up the array's address (make it outside graph capture).  All calls on
 * one GPU share the array: calls that overlap on one GPU (two streams, two threads) race on it.  Nothing in it
 * has to be cleared between calls: a merge reads only partials that the same call has written.
 */
#define MVLLM_PAGED_DECODE_NOALLOC_MAX_BYTES (32u << 20)
int mvllm_paged_decode_noalloc(void* out, const void* q,
                               const void* k_cache, const void* v_cache,
                               const int32_t* block_tables, int max_num_blocks,
                               const void* context_lens, int ctx_is_i64,
                               int batch, int num_heads, int num_kv_heads, int head_dim,
                               int block_size, int64_t num_blocks, float scale, int dtype,
                               void* stream);

/*
 * flash_attention_prefill -- src/myvllm/layers/attention.py:212-280 (kernel :111-209).
 * Packed ragged batch: sequence s owns rows [cu_seqlens[s], cu_seqlens[s+1]).
 * out[i,h,:] = softmax_{j<=i, same sequence}( scale * q[i,h,:] . k[j,g(h),:] ) v[j,g(h),:].
 *   out, q  [T, Hq, D];  k, v  [T, Hkv, D];  cu_seqlens int32 [num_seqs+1]
 * Needs no maximum sequence length: the grid is sized from total_tokens and
 * num_seqs (the reference synchronises with the host to find it, :263-264).
 */
int mvllm_prefill_varlen(void* out, const void* q, const void* k, const void* v,
                         const int32_t* cu_seqlens, int num_seqs, int64_t total_tokens,
                         int num_heads, int num_kv_heads, int head_dim,
                         float scale, int dtype, void* stream);

/*
 * Which kernel a prefill of these static sizes runs on (no counterpart in the reference, whose Triton kernels take any
 * power-of-two head_dim from a tile-size table, attention.py:249-257).  block_size 0 = the packed entry point,
 * > 0 = the paged ones.  *kernel: 2 an LDS-tiled MFMA kernel (bf16 / fp16 with a head_dim that is a multiple of 8 from
 * 32 to 128, or 256; fp32 with 128 or 64; over an INT8 cache 64 or 128; the packed and the 16-bit paged entry point run its
 * two-group form where head_dim is 128, the query heads per kv head are an even number and the batch has at most 64
 * sequences), 1 the 16-row tile MFMA kernel (a paged cache whose blocks hold 2^31 bytes or more), 0 the generic kernel (any
 * head_dim <= 512; one key per step, a correctness path two orders of magnitude slower), -1 unsupported.
 * Pointers are assumed 16-byte aligned (unaligned ones take the generic kernel).  Pure host arithmetic.
 */
int mvllm_prefill_plan(int num_heads, int num_kv_heads, int head_dim, int block_size, int dtype,
                       int int8_cache, int* kernel);

/*
 * Prefill over a paged cache: the same attention as mvllm_prefill_varlen for sequences whose first tokens are
 * already in the cache (prefix-cache hits).  The reference prepares exactly this metadata in
 * ModelRunner.prepare_prefill (src/myvllm/engine/model_runner.py:192-226: input_ids = tokens[num_cached:],
 * cu_seqlens_q over the new tokens, cu_seqlens_k over all of them, block_tables when they differ) but its
 * Attention.forward never consumes it (attention.py:518-523 passes cu_seqlens_q and the fresh k, v only).
 *   q, out       [total_q_tokens, Hq, D]: rows of the new tokens only, packed by cu_seqlens_q
 *   k/v_cache    [num_blocks, block_size, Hkv, D], already holding every key of every sequence
 *                (prefix from earlier requests, new tokens from the store that precedes this call)
 *   block_tables int32 [num_seqs, max_num_blocks]; cu_seqlens_q/k int32 [num_seqs+1]
 * Query row r of sequence s (r counted over its new tokens) sits at position
 * c_s + r, c_s = len_k(s) - len_q(s), and attends keys 0 .. c_s + r.  The first ceil(len_k/bs) table
 * entries of a sequence are expected to be valid; an entry < 0 or >= num_blocks there is not followed (no
 * out-of-range access): its keys and values read as zeros.  With c_s = 0 for every s the result equals
 * mvllm_prefill_varlen bit for bit (block sizes that are multiples of 16: both calls then run the same kernel).
 */
int mvllm_prefill_paged(void* out, const void* q, const void* k_cache, const void* v_cache,
                        const int32_t* block_tables, int max_num_blocks,
                        const int32_t* cu_seqlens_q, const int32_t* cu_seqlens_k,
                        int num_seqs, int64_t total_q_tokens,
                        int num_heads, int num_kv_heads, int head_dim, int block_size,
                        int64_t num_blocks, float scale, int dtype, void* stream);

/*
 * The same prefill over an INT8 cache (codes + fp32 scales per (token, kv head), as mvllm_store_kvcache_int8 writes
 * them; no counterpart in the reference, which has neither an INT8 cache nor a consumer of its prefix-cache
 * metadata).  Every key, the new tokens' included, is read from the cache and dequantised (code * scale, rounded
 * to `dtype`) on the way into the matrix unit, which is what decode will see for the same tokens.
 * bf16 / fp16 queries, head_dim 128 or 64, block_size a multiple of 16; else MVLLM_ERR_UNSUPPORTED.
 */
int mvllm_prefill_paged_int8(void* out, const void* q,
                             const int8_t* k_cache, const int8_t* v_cache,
                             const float* k_scale, const float* v_scale,
                             const int32_t* block_tables, int max_num_blocks,
                             const int32_t* cu_seqlens_q, const int32_t* cu_seqlens_k,
                             int num_seqs, int64_t total_q_tokens,
                             int num_heads, int num_kv_heads, int head_dim, int block_size,
                             int64_t num_blocks, float scale, int dtype, void* stream);

/*
 * mvllm_prefill_paged and mvllm_prefill_paged_int8 in two steps, for callers that can lend device memory: every
 * sequence's keys and values are first written into `workspace`, laid out as a 16-bit paged cache of 16-token blocks with
 * a block table of its own, and the two-group prefill kernel (shapes it does not take: the one-group kernel's 16-bit
 * paged form) runs over that.  No counterpart in the reference.  Two uses:
 *   - an INT8 cache: a value is dequantised once (the same code * scale rounded to `dtype`), where the one-step form
 *     converts a K/V tile again for every query tile that walks it;
 *   - any block_size >= 1: the one-step forms need a multiple of 16 for their MFMA kernels.
 *   max_kv_len     an upper bound of every sequence's len_k, known to the host (the reference's Context.max_seqlen_k,
 *                  utils/context.py:11); keys of a sequence past it read as zeros
 *   workspace      256-byte aligned, at least mvllm_prefill_paged_staged_workspace_bytes(...) bytes; contents need not
 *                  be kept between calls; calls that share a workspace must not overlap
 * mvllm_prefill_paged_staged_workspace_bytes returns 0 for shapes this form is not built for (it takes bf16 / fp16 with
 * head_dim 128 or 64, 16-bit caches also 32, 48, 80, 96, 112 and 256); the entry points then return
 * MVLLM_ERR_UNSUPPORTED and the one-step form is the one to call.
 * Other arguments and the result's meaning as for the one-step forms; MVLLM_ERR_WORKSPACE for a workspace that is null,
 * too small or misaligned.
 */
size_t mvllm_prefill_paged_staged_workspace_bytes(int num_seqs, int max_kv_len, int num_heads, int num_kv_heads,
                                                  int head_dim, int dtype, int int8_cache);
int mvllm_prefill_paged_staged(void* out, const void* q, const void* k_cache, const void* v_cache,
                               const int32_t* block_tables, int max_num_blocks,
                               const int32_t* cu_seqlens_q, const int32_t* cu_seqlens_k,
                               int num_seqs, int64_t total_q_tokens, int max_kv_len,
                               int num_heads, int num_kv_heads, int head_dim, int block_size,
                               int64_t num_blocks, float scale, int dtype,
                               void* workspace, size_t workspace_bytes, void* stream);
int mvllm_prefill_paged_int8_staged(void* out, const void* q,
                                    const int8_t* k_cache, const int8_t* v_cache,
                                    const float* k_scale, const float* v_scale,
                                    const int32_t* block_tables, int max_num_blocks,
                                    const int32_t* cu_seqlens_q, const int32_t* cu_seqlens_k,
                                    int num_seqs, int64_t total_q_tokens, int max_kv_len,
                                    int num_heads, int num_kv_heads, int head_dim, int block_size,
                                    int64_t num_blocks, float scale, int dtype,
                                    void* workspace, size_t workspace_bytes, void* stream);

/*
 * mvllm_prefill_paged with every sequence's keys cut into `splits` ranges that are walked side by side and merged: for
 * batches of few new tokens behind long cached prefixes (a follow-up turn, the last chunk of a chunked prefill), whose
 * few query tiles would each walk a whole prefix while most of the chip idles.  No counterpart in the reference (its
 * prefill never reads the paged cache, src/myvllm/layers/attention.py:111-209, and the prefix-hit metadata that
 * model_runner.py:192-226 builds goes unused, attention.py:518-523).
 * 16-bit caches at the head dims of the LDS-tiled kernel (64, 128; 32, 48, 80, 96, 112, 256), INT8 caches
 * (mvllm_prefill_paged_int8_split: codes + scales as for mvllm_prefill_paged_int8) at head_dim 64 and 128; block_size a
 * multiple of 16, num_seqs * splits <= 64.
 *   _split_plan: the number of ranges the library would use for a batch of these sizes; 0 = run mvllm_prefill_paged.
 *   _split_workspace_bytes: 256-byte aligned device memory the call needs for `splits` ranges (range tables, partial
 *     results [splits, total_q_tokens, Hq, D] and their softmax denominators); 0 = shape not taken.
 * max_kv_len: the host's upper bound of every sequence's key count, as in the staged forms.  Results differ from the
 * one-step form's by the rounding of the partial results to the element type (within the same tolerance).
 */
int mvllm_prefill_paged_split_plan(int num_seqs, int64_t total_q_tokens, int max_kv_len, int num_heads,
                                   int num_kv_heads, int head_dim, int block_size, int dtype, int int8_cache);
size_t mvllm_prefill_paged_split_workspace_bytes(int num_seqs, int64_t total_q_tokens, int max_kv_len, int num_heads,
                                                 int num_kv_heads, int head_dim, int block_size, int dtype, int splits);
int mvllm_prefill_paged_split(void* out, const void* q, const void* k_cache, const void* v_cache,
                              const int32_t* block_tables, int max_num_blocks,
                              const int32_t* cu_seqlens_q, const int32_t* cu_seqlens_k,
                              int num_seqs, int64_t total_q_tokens, int max_kv_len,
                              int num_heads, int num_kv_heads, int head_dim, int block_size,
                              int64_t num_blocks, float scale, int dtype, int splits,
                              void* workspace, size_t workspace_bytes, void* stream);
int mvllm_prefill_paged_int8_split(void* out, const void* q,
                                   const int8_t* k_cache, const int8_t* v_cache,
                                   const float* k_scale, const float* v_scale,
                                   const int32_t* block_tables, int max_num_blocks,
                                   const int32_t* cu_seqlens_q, const int32_t* cu_seqlens_k,
                                   int num_seqs, int64_t total_q_tokens, int max_kv_len,
                                   int num_heads, int num_kv_heads, int head_dim, int block_size,
                                   int64_t num_blocks, float scale, int dtype, int splits,
                                   void* workspace, size_t workspace_bytes, void* stream);

/*
 * The caller's per-layer chain between the QKV projection and the attention kernels, fused:
 *   q = rms_norm(q); k = rms_norm(k)      src/myvllm/models/qwen3.py:104-106, layers/layernorm.py:9-17
 *   q, k = rotary_emb(positions, q, k)    qwen3.py:108, layers/rotary_embedding.py:4-23, 77-83
 *   store_kvcache(k, v, ...)              layers/attention.py:67-108 (called from Attention.forward :505-506)
 * q, k, v are rows of num_heads*D / num_kv_heads*D / num_kv_heads*D elements with the given strides (in
 * elements) between tokens, so the three slices of the packed QKV projection output can be passed as they
 * lie.  gamma [D] fp32 is the shared RMSNorm weight (NULL: no norm, the reference's qkv_bias=True case);
 * cos_sin_cache [max_position, D] fp32 holds cos (D/2) then sin (D/2) per position (rotary_embedding.py:61-70);
 * positions int64 [T] are clamped to [0, max_position).  Rotation pairs element i with i + D/2.
 * Rounding follows the unfused chain: norm result rounded to the element type, rotation in fp32 on the
 * rounded values, rounded again.
 * Outputs: q_out [T, Hq, D] always; k_out / v_out [T, Hkv, D] when not NULL (the prefill kernel reads them);
 * when slot_mapping is not NULL the rotated k and v go to flat slot slot_mapping[t] of the caches
 * (slots < 0 or >= num_slots skipped): element-type caches, or with cache_is_int8 != 0 int8 codes and
 * fp32 scales exactly as mvllm_store_kvcache_int8 would write them from k_out / v.
 * head_dim % 8 == 0, head_dim <= 512; 8-byte aligned pointers (16-byte for fp32), strides % 4 == 0.
 */
int mvllm_qk_norm_rope_store(void* q_out, void* k_out, void* v_out,
                             const void* q, const void* k, const void* v,
                             int64_t q_row_stride, int64_t k_row_stride, int64_t v_row_stride,
                             const float* gamma, float eps,
                             const float* cos_sin_cache, int64_t max_position,
                             const int64_t* positions, const int64_t* slot_mapping,
                             void* k_cache, void* v_cache, float* k_scale, float* v_scale, int cache_is_int8,
                             int64_t num_tokens, int64_t num_slots,
                             int num_heads, int num_kv_heads, int head_dim, int dtype, void* stream);

/*
 * SamplerLayer.forward -- src/myvllm/layers/sampler.py:14-19:
 *   logits /= temperature; probs = softmax(logits); token = argmax(probs / exponential_(1).clamp_min_(1e-10))
 * One launch, no (batch, vocab) probability tensor: out_ids[b] = argmax_i( logits[b,i] / temperatures[b]
 * - log(max(E[b,i], 1e-10)) ), which is the same argmax (softmax only rescales a row by a positive factor).
 * Ties go to the smallest index.
 *   logits        [batch, vocab] in dtype, row_stride elements between rows (the LM-head GEMM output as it lies)
 *   temperatures  fp32 [batch], > 0
 *   noise         fp32 [batch, vocab] of Exp(1) draws, or NULL: then E comes from Philox4x32-10 with key = seed
 *                 and counter = (i / 4, b, offset): lane (i % 4) of the output word gives u = ((x >> 8) + 0.5) * 2^-24
 *                 and E = -log(u).  Advance `offset` by one per call for independent draws.
 *   out_ids       int64 [batch]
 *   workspace     optional scratch of mvllm_sample_tokens_workspace_bytes(batch, vocab) bytes: with it a row is
 *                 scanned by several workgroups (a small batch alone cannot occupy the GPU) and a second tiny
 *                 launch picks the winner; NULL or too small: one workgroup per row, same result.
 */
size_t mvllm_sample_tokens_workspace_bytes(int batch, int vocab);
int mvllm_sample_tokens(int64_t* out_ids, const void* logits, int64_t row_stride,
                        const float* temperatures, const float* noise,
                        uint64_t seed, uint64_t offset, int batch, int vocab, int dtype,
                        void* workspace, size_t workspace_bytes, void* stream);

/*
 * mvllm_sample_tokens with in-kernel noise whose call offset is read from device memory (*offset_dev), for a
 * sampler inside a captured graph: a replay cannot change a launch argument, the graph increments the counter.
 */
int mvllm_sample_tokens_dev_offset(int64_t* out_ids, const void* logits, int64_t row_stride,
                                   const float* temperatures, uint64_t seed, const uint64_t* offset_dev,
                                   int batch, int vocab, int dtype,
                                   void* workspace, size_t workspace_bytes, void* stream);

/*
 * LM head + sampler in one pass over the weights -- ParallelLMHead.forward (src/myvllm/layers/embedding_head.py:56-77:
 * rows to sample from, hidden W^T) followed by SamplerLayer.forward (layers/sampler.py:14-19), without the
 * (batch, vocab) logits reaching memory:
 *   out_ids[b] = argmax_n( bf16(hidden[row_index[b]] . W[n]) / T[b] - log(max(E[b, n], 1e-10)) )
 * with the logit rounded to the element type, as the materialised tensor would be, and E drawn as in
 * mvllm_sample_tokens (Philox4x32-10, key = seed, counter = (n / 4, b, offset (+ *offset_dev when not NULL))): the
 * same ids as mvllm_sample_tokens on the rounded product, up to the order of the fp32 sums inside a logit.
 * hidden rows hidden_row_stride elements apart (a multiple of 8); row_index int64 [batch] or NULL (rows 0..batch-1:
 * a decode step; the last token of every packed sequence in prefill, embedding_head.py:57-62); weight [vocab, K]
 * dense.  batch <= 64, vocab % 16 == 0, K in {256, 512, 1024}, bf16 / fp16; otherwise MVLLM_ERR_UNSUPPORTED and the
 * caller runs the library GEMM and mvllm_sample_tokens.  workspace: mvllm_lm_head_sample_workspace_bytes(batch, K)
 * bytes, 8-byte aligned, caller-owned.  The first launch of a shape with more than 48 KB of hidden rows raises the
 * kernel's dynamic LDS limit (a host-side attribute call: make it outside a graph capture).
 */
size_t mvllm_lm_head_sample_workspace_bytes(int batch, int K);
int mvllm_lm_head_sample(int64_t* out_ids, const void* hidden, int64_t hidden_row_stride,
                         const int64_t* row_index, const void* weight, const float* temperatures,
                         uint64_t seed, uint64_t offset, const uint64_t* offset_dev, int batch, int vocab,
                         int K, int dtype, void* workspace, size_t workspace_bytes, void* stream);

/*
 * The step metadata of a decode batch that continues the step before it (same sequences, each one token longer),
 * advanced on the device in one launch instead of being rebuilt on the host as ModelRunner.prepare_decode does
 * (src/myvllm/engine/model_runner.py:231-256): input_ids[i] = sampled[i]; context_lens[i] += 1;
 * positions[i] = context_lens[i] - 1; slot_mapping[i] += 1.  All int64 [batch].  Rows whose context length is
 * not positive (the padding of a captured batch size) are left alone.  Rows that open a new block have their slot
 * and table entry patched by the caller afterwards.  step_counter (may be NULL): one uint64 on the device, the
 * call counter of mvllm_sample_tokens_dev_offset / mvllm_lm_head_sample, incremented by one, so that a captured
 * decode step can end with this launch and be replayed without any host-side update.  host_ids (may be NULL; needs
 * step_counter): two rows of host_row_stride >= batch + 1 int64 in pinned, device-visible host memory; row
 * (counter before the increment) & 1 receives sampled[0 .. batch) and then, behind a system-scope fence, the new
 * counter value in its last entry: the host reads a step's ids once it sees that value, with no copy operation and
 * no event queued between two replays (two rows: step t is read while step t + 1 runs).
 */
int mvllm_decode_advance(int64_t* input_ids, int64_t* context_lens, int64_t* positions, int64_t* slot_mapping,
                         const int64_t* sampled, uint64_t* step_counter, int64_t* host_ids,
                         int64_t host_row_stride, int batch, void* stream);

/*
 * LayerNorm.forward with and without residual -- src/myvllm/layers/layernorm.py:9-28, called from
 * Qwen3DecoderLayer.forward and the final norm (src/myvllm/models/qwen3.py:197-212, 306-312):
 *   x = x + residual (rounded to the element type);  out = x / sqrt(mean(x^2) + eps) * gamma;  residual_out = x
 * x [rows, hidden] with x_row_stride elements between rows; residual likewise or NULL (no add);
 * residual_out [rows, hidden] dense or NULL; out [rows, hidden] dense; gamma fp32 [hidden].
 * hidden % 8 == 0, hidden <= 8192, 16-byte aligned pointers, strides % 8 == 0.
 */
int mvllm_add_rms_norm(void* out, void* residual_out, const void* x, const void* residual,
                       const float* gamma, float eps, int64_t rows, int hidden,
                       int64_t x_row_stride, int64_t residual_row_stride, int dtype, void* stream);

/*
 * SiluAndMul.forward -- src/myvllm/layers/activation.py:15-18:  x, y = in.chunk(2, -1); out = silu(x) * y
 * in [rows, 2*width] with in_row_stride elements between rows; out [rows, width] dense.  silu(x) is rounded to
 * the element type before the product, as the two tensor operations would.  width a multiple of 16 bytes.
 */
int mvllm_silu_and_mul(void* out, const void* in, int64_t rows, int width, int64_t in_row_stride,
                       int dtype, void* stream);

/*
 * The caller's projections around the attention path for the few rows of a decode step -- nn.Linear in
 * src/myvllm/models/qwen3.py:90-94 (QKV), :118 (output projection) and the MLP (:121-160; layers/linear.py):
 *   out[M, N] = x[M, K] W[N, K]^T + bias[N]
 * M <= 64, bf16 / fp16 with fp32 accumulation, N % 16 == 0, K % 512 == 0; x rows x_row_stride elements apart
 * (a multiple of 8), W dense, bias in the element type or NULL; x and W 16-byte aligned.  Larger M (prefill) stays
 * a library GEMM: MVLLM_ERR_UNSUPPORTED.
 */
int mvllm_linear_small_m(void* out, const void* x, const void* w, const void* bias, int64_t x_row_stride,
                         int M, int N, int K, int dtype, void* stream);

/*
 * The same product with the launches around it folded in, for the decoder layer's decode step
 * (src/myvllm/models/qwen3.py:197-212: residual add + RMSNorm, projection; :151-160: gate/up, SiluAndMul):
 *   gamma != NULL:  h = x + residual (rounded to the element type; residual NULL: h = x), residual_out = h (may be
 *                   NULL), x' = h / sqrt(mean(h^2) + eps) * gamma rounded to the element type, exactly what
 *                   mvllm_add_rms_norm writes (layers/layernorm.py:9-28) up to the order of the sum of squares;
 *                   the product is taken of x'.  residual and residual_out are dense [M, K]; residual_out must not
 *                   alias x or residual (every workgroup reads all of both while one of them writes a row).
 *   glu != 0:       W is [2F, K] (gate rows, then up rows, as layers/activation.py:15-18 chunks the output), out is
 *                   [M, F] = silu(x' Wg^T + bg) * (x' Wu^T + bu) with the roundings of mvllm_silu_and_mul on the
 *                   rounded projection; N = 2F, N % 32 == 0.
 * Shapes as mvllm_linear_small_m, and for gamma != NULL: N / 16 >= min(M, 16), K / waves one burst of 128 or 256
 * values with 4, 8 or 16 waves (mvllm_linear_small_m_plan says whether a shape is taken); otherwise MVLLM_ERR_UNSUPPORTED and the caller
 * runs the separate launches.
 */
int mvllm_norm_linear_small_m(void* out, void* residual_out, const void* x, const void* residual,
                              const float* gamma, float eps, const void* w, const void* bias,
                              int64_t x_row_stride, int M, int N, int K, int glu, int dtype, void* stream);

/*
 * Whether mvllm_linear_small_m (norm == 0 && glu == 0) or mvllm_norm_linear_small_m takes a shape, without a
 * launch: MVLLM_OK and the waves per workgroup in *waves (may be NULL), or MVLLM_ERR_UNSUPPORTED.  No counterpart
 * in the reference (its projections are library GEMMs of any shape).
 */
int mvllm_linear_small_m_plan(int M, int N, int K, int norm, int glu, int dtype, int* waves);

/*
 * Attention with a sink: the four calls below are mvllm_paged_decode, mvllm_prefill_varlen, mvllm_prefill_paged and
 * mvllm_prefill_paged_split with one more term in every softmax denominator, exp(sink[h]): a learned number per query
 * head that has neither key nor value and is not scaled (no counterpart in the reference).  sink fp32 [Hq] on the device.
 * The prefill forms run on the one-group, fp32 and generic kernels; a paged cache whose blocks hold 2^31 bytes or more
 * is MVLLM_ERR_UNSUPPORTED.
 */
int mvllm_paged_decode_sink(void* out, const void* q, const void* k_cache, const void* v_cache,
                            const int32_t* block_tables, int max_num_blocks, const void* context_lens, int ctx_is_i64,
                            int batch, int num_heads, int num_kv_heads, int head_dim, int block_size,
                            int64_t num_blocks, float scale, const float* sink, int dtype, void* workspace,
                            size_t workspace_bytes, void* stream);
int mvllm_prefill_varlen_sink(void* out, const void* q, const void* k, const void* v, const int32_t* cu_seqlens,
                              int num_seqs, int64_t total_tokens, int num_heads, int num_kv_heads, int head_dim,
                              float scale, const float* sink, int dtype, void* stream);
int mvllm_prefill_paged_sink(void* out, const void* q, const void* k_cache, const void* v_cache,
                             const int32_t* block_tables, int max_num_blocks, const int32_t* cu_seqlens_q,
                             const int32_t* cu_seqlens_k, int num_seqs, int64_t total_q_tokens, int num_heads,
                             int num_kv_heads, int head_dim, int block_size, int64_t num_blocks, float scale,
                             const float* sink, int dtype, void* stream);
int mvllm_prefill_paged_split_sink(void* out, const void* q, const void* k_cache, const void* v_cache,
                                   const int32_t* block_tables, int max_num_blocks, const int32_t* cu_seqlens_q,
                                   const int32_t* cu_seqlens_k, int num_seqs, int64_t total_q_tokens, int max_kv_len,
                                   int num_heads, int num_kv_heads, int head_dim, int block_size, int64_t num_blocks,
                                   float scale, const float* sink, int dtype, int splits, void* workspace,
                                   size_t workspace_bytes, void* stream);

/*
 * Between two sublayers that have a norm on either side and a short causal convolution in front (no counterpart in the
 * reference; the residual stream is fp32):
 *     x' = x + rms(y) * post;   h = rms(x') * pre;   out_t = h_t + sum_j conv[j] * h_(t - taps + 1 + j)
 *   out      [rows, width] dtype;  x_out fp32 [rows, width] = x' or NULL (must not be x)
 *   x        fp32 [rows, width], or NULL with embed [vocab, width] dtype and tokens int64 [rows] (x = embed[token])
 *   y        [rows, width] dtype or NULL (x' = x);  post, pre: fp32 gains, one number (stride 0) or [width] (stride 1)
 *   conv     fp32 [taps, width] or NULL (out = h), taps 1 .. 8;  state fp32 [num_banks, taps - 1, width]: the last
 *            taps - 1 rows of h, read before an entry's first row (zeros before position 0) and written after its last
 *   cu_seqlens int32 [entries + 1] rows of the entries (all rows covered), row_entry int32 [rows], bank_in / bank_out
 *            int32 [entries] (they must differ for entries of more than one row), positions int64 [rows]
 * bf16 and fp32, width up to 16384 (4096 where it is not a multiple of 4).
 */
int mvllm_norm_conv(void* out, float* x_out, const float* x, const void* embed, const int64_t* tokens, int64_t vocab,
                    const void* y, const float* post, int post_stride, const float* pre, int pre_stride, float eps,
                    const float* conv, int taps, float* state, int64_t num_banks, const int32_t* cu_seqlens,
                    const int32_t* row_entry, const int32_t* bank_in, const int32_t* bank_out, const int64_t* positions,
                    int64_t rows, int width, int dtype, void* stream);

/*
 * Per-head norms, rotary embedding in either pair layout, rotated values and the cache store for heads whose key and
 * value sizes may differ (models/qwen3.py:104-110 is the reference's case of it).
 *   proj [rows, proj_row_stride]: q [Hq, dim] | k [Hkv, dim] | v [Hkv, vdim] | anything
 *   q_out [*, Hq, head_dim], k_out / v_out [*, Hkv, head_dim] or NULL: row dst_row[t] (NULL: t); dims past dim / vdim
 *   are zeros.  k_cache / v_cache [num_slots, Hkv, head_dim] rows slots[t] (< 0 or NULL: none).
 *   gain_q / gain_k fp32 [dim] or NULL (no norm); q_scale multiplies q last.
 *   rot_table fp32 [max_position, rot_dims / 2, 2], v_table fp32 [max_position, vdim / 2, 2] or NULL: (cos, sin) per
 *   pair; interleaved: pair i is dims 2i, 2i + 1, else i, i + n / 2.
 * bf16 and fp32, head_dim up to 512.
 */
int mvllm_head_rope_store(void* q_out, void* k_out, void* v_out, const void* proj, int64_t proj_row_stride,
                          const float* gain_q, const float* gain_k, float eps, float q_scale, const float* rot_table,
                          int rot_dims, const float* v_table, int interleaved, int64_t max_position,
                          const int64_t* positions, const int32_t* dst_row, const int64_t* slots, void* k_cache,
                          void* v_cache, int64_t num_slots, int64_t rows, int num_heads, int num_kv_heads, int dim,
                          int vdim, int head_dim, int dtype, void* stream);

/*
 * mvllm_head_rope_store with other norms, added up in `norms`: 1: q and k over all heads of a row at once (gain_q fp32 [Hq dim],
 * gain_k [Hkv dim]) in front of the rotation; 2: q and k of every head divided by their root mean square behind it; 4: values
 * divided by theirs (behind a rotation, if there is one).  head_scale fp32 [Hq] or NULL: a further factor of q.  kv_row int64
 * [rows] or NULL: rows of k_out and v_out (< 0: none).  kv_head_stride: elements between the heads of a row of k_out, v_out and
 * the caches (with v_cache = k_cache + head_dim and twice head_dim, a key and its value are neighbours).
 */
int mvllm_head_norm_rope_store(void* q_out, void* k_out, void* v_out, const int64_t* kv_row, const void* proj,
                               int64_t proj_row_stride, const float* gain_q, const float* gain_k, int norms, float eps,
                               float q_scale, const float* head_scale, const float* rot_table, int rot_dims,
                               const float* v_table, int interleaved, int64_t max_position, const int64_t* positions,
                               const int32_t* dst_row, const int64_t* slots, void* k_cache, void* v_cache, int kv_head_stride,
                               int64_t num_slots, int64_t rows, int num_heads, int num_kv_heads, int dim, int vdim,
                               int head_dim, int dtype, void* stream);

/*
 * Behind attention over rotated values: out[t, h, :vdim] = rotate(o[dst_row[t], h], -position) * sigmoid(gate[t, h]).
 * o [*, Hq, head_dim]; gate [rows, gate_row_stride] dtype, Hq values per row, or NULL; v_table as above or NULL.
 */
int mvllm_head_unrotate_gate(void* out, const void* o, const void* gate, int64_t gate_row_stride, const float* v_table,
                             int interleaved, int64_t max_position, const int64_t* positions, const int32_t* dst_row,
                             int64_t rows, int num_heads, int vdim, int head_dim, int dtype, void* stream);

/*
 * Decode metadata of a cache that holds one attention chunk per sequence (chunk 0: the whole sequence): for a row with
 * context length c > 0, chunk_lens = (c - 1) mod chunk + 1 and slots = the slot of that last token; 0 and -1 otherwise.
 * All int64 [batch] but block_tables int32 [batch, max_num_blocks].
 */
int mvllm_chunk_decode_step(int64_t* chunk_lens, int64_t* slots, const int64_t* context_lens,
                            const int32_t* block_tables, int max_num_blocks, int chunk, int block_size, int batch,
                            void* stream);

/*
 * out[rows, N] (fp32) = act(x W^T + bias): columns below `split` get cap * tanh(z / cap) (cap 0: z), the others
 * logsigmoid of that.  x [rows, K], w [N, K] dtype; bias fp32 [N] or NULL.  For the gates of a recurrence, N small.
 */
int mvllm_gate_linear(float* out, const void* x, int64_t x_row_stride, const void* w, const float* bias, int64_t rows,
                      int N, int K, int split, float cap, int dtype, void* stream);

/*
 * mLSTM matrix-memory recurrence (csrc/mlstm.hip has the equations): every row of every entry in turn.
 *   num fp32 [rows, H, vdim], den fp32 [rows, H] (the floor added), m_next fp32 [entries, H]
 *   proj [rows, proj_row_stride]: q [H, dim] | k [H, dim] | v [H, vdim] | anything;  gates fp32 [rows, 2 H]
 *   state of slot slots[e]: s_state fp32 [*, H, dim, vdim], n_state [*, H, dim], m_state [*, H]; s and n are updated,
 *   m by mvllm_mlstm_output; an entry that starts at position 0 starts from zeros.  slots < 0: the entry is skipped.
 * mvllm_mlstm_output: out [rows, H * vdim] = rms(num / den) * weight * sigmoid(gate), m_state[slot] = m_next.
 * mvllm_mlstm_chunked: the recurrence's results for entries of many rows in blocks of 64 rows on the matrix unit (bf16,
 *   dim <= 256, dim and vdim multiples of 8; others: MVLLM_ERR_UNSUPPORTED).  segments int32 [num_segments, 4]: entry,
 *   first row, rows, flags (1 first, 2 last, 4 the only one of its entry), the segments of an entry in order and next to
 *   each other, all but the last a multiple of 64 rows.  split != 0 (some entry has several): workspace of
 *   mvllm_mlstm_chunked_workspace_bytes.
 */
int mvllm_mlstm_recurrent(float* num, float* den, float* m_next, const void* proj, int64_t proj_row_stride,
                          const float* gates, float* s_state, float* n_state, const float* m_state,
                          const int32_t* cu_seqlens, const int32_t* slots, const int64_t* positions, int entries,
                          int num_heads, int dim, int vdim, float q_scale, float floor, int dtype, void* stream);
size_t mvllm_mlstm_chunked_workspace_bytes(int num_segments, int num_heads, int dim, int vdim);
int mvllm_mlstm_chunked(float* num, float* den, float* m_next, const void* proj, int64_t proj_row_stride,
                        const float* gates, float* s_state, float* n_state, const float* m_state,
                        const int32_t* cu_seqlens, const int32_t* slots, const int64_t* positions,
                        const int32_t* segments, int num_segments, int split, int num_heads, int dim, int vdim,
                        float q_scale, float floor, int dtype, void* workspace, size_t workspace_bytes, void* stream);
int mvllm_mlstm_output(void* out, const float* num, const float* den, const float* weight, const void* gate,
                       int64_t gate_row_stride, float eps, const float* m_next, float* m_state,
                       const int32_t* cu_seqlens, const int32_t* row_entry, const int32_t* slots, int64_t rows,
                       int num_heads, int vdim, int dtype, void* stream);

/*
 * Between two sublayers of a decoder whose residual is `streams` fp32 streams (hyper-connections; csrc/stream_norm.hip):
 *     y' = scale * y;   x'_t = sum_s mix[s, t] x_s + out[t] y';   h = rms(sum_t in[t] x'_t) * gain
 *   out [rows, out_row_stride] dtype = h, zeros past width;  x_out fp32 [rows, streams, width] = x' or NULL (may be x)
 *   x fp32 [rows, streams, width];  scale fp32 [width] or NULL;  hc_out [streams], hc_mix [streams, streams] (from x to),
 *   hc_in [streams] or NULL (the plain sum), gain [width]: fp32
 *   y: [rows, y_row_stride] dtype, or with parts: y = sum_k weights[t, k] parts[part_row[t, k]] + sigmoid(gate[t]) * y,
 *   parts [*, part_row_stride] dtype, part_row int32 [rows, top] (NULL: row t * top + k), weights fp32 [rows, top],
 *   gate fp32, one per row gate_row_stride apart (NULL: 1), y NULL: no such row.
 * mvllm_stream_embed_norm starts the streams: x_s = embed[token] * embed_scale + bigram[b], b = (previous * mul_prev +
 *   token * mul_cur) mod buckets, b = buckets for a sequence's first token; embed [vocab, width], bigram [buckets + 1, width]
 *   or NULL.  The token before an entry's first row is prev_tokens[bank_in[entry]] (int64); its last row writes
 *   prev_tokens[bank_out[entry]].  Banks must differ for entries of more than one row.
 * bf16 and fp32, up to 8 streams, width up to 16384 (4096 where it is not a multiple of 4).
 */
int mvllm_stream_embed_norm(void* out, int64_t out_row_stride, float* x_out, const void* embed, int64_t vocab,
                            float embed_scale, const void* bigram, int64_t buckets, int64_t mul_prev, int64_t mul_cur,
                            int64_t* prev_tokens, const int64_t* tokens, const int64_t* positions,
                            const int32_t* cu_seqlens, const int32_t* row_entry, const int32_t* bank_in,
                            const int32_t* bank_out, const float* hc_in, const float* gain, float eps, int64_t rows,
                            int streams, int width, int dtype, void* stream);
int mvllm_stream_norm(void* out, int64_t out_row_stride, float* x_out, const float* x, const void* y, int64_t y_row_stride,
                      const void* parts, int64_t part_row_stride, const int32_t* part_row, const float* weights, int top,
                      const float* gate, int64_t gate_row_stride, const float* scale, const float* hc_out,
                      const float* hc_mix, const float* hc_in, const float* gain, float eps, int64_t rows, int streams,
                      int width, int dtype, void* stream);

/*
 * Matrix memory with a constant decay per head: S = decay S + k v^T, num = S^T q (csrc/decay_memory.hip).
 *   proj [rows, proj_row_stride]: q [H, dim] | k [H, dim] | v [H, vdim] | anything; silu != 0: each through z sigmoid(z)
 *   num fp32 [rows, H, vdim];  decay fp32 [H] (the chunked form: its natural logarithm);  s_state fp32 [*, H, dim, vdim]
 *   everything else as for mvllm_mlstm_recurrent / mvllm_mlstm_chunked.
 * mvllm_gated_row_norm: out [rows, out_row_stride] = rms(x) * weight * sigmoid(gate), zeros past width; x fp32 [rows, width].
 */
int mvllm_decay_memory_recurrent(float* num, const void* proj, int64_t proj_row_stride, const float* decay, float* s_state,
                                 const int32_t* cu_seqlens, const int32_t* slots, const int64_t* positions, int entries,
                                 int num_heads, int dim, int vdim, int silu, int dtype, void* stream);
size_t mvllm_decay_memory_chunked_workspace_bytes(int num_segments, int num_heads, int dim, int vdim);
int mvllm_decay_memory_chunked(float* num, const void* proj, int64_t proj_row_stride, const float* log_decay,
                               float* s_state, const int32_t* cu_seqlens, const int32_t* slots, const int64_t* positions,
                               const int32_t* segments, int num_segments, int split, int num_heads, int dim, int vdim,
                               int silu, int dtype, void* workspace, size_t workspace_bytes, void* stream);
int mvllm_gated_row_norm(void* out, int64_t out_row_stride, const float* x, const float* weight, const void* gate,
                         int64_t gate_row_stride, float eps, int64_t rows, int width, int dtype, void* stream);

/*
 * Attention over latents (csrc/latent.hip): a cache of one row per token, `padded` (a multiple of 32) elements wide with
 * zeros past the rank.
 * mvllm_latent_norm_store: c = rms(in[:rank]) * weight -> out [rows, padded] (or NULL) and cache row slots[t] (< 0: none).
 * mvllm_head_linear: out[t, h, :N] = W_h x[t, h, :K], w [H, N, K]; row and head strides in elements.  bf16: K % 8 == 0,
 *   N % 16 == 0.
 * mvllm_latent_decode: softmax(scale q . c) c over the first lens[t] (int64) rows of entry row_entry[t]'s table: q and out
 *   [rows, H, padded], cache [num_blocks, block_size, padded], block_tables int32 [entries, table_width]; 0 keys: zeros.
 *   workspace: mvllm_latent_decode_workspace_bytes (max_keys = table_width * block_size), 16-byte aligned.
 */
int mvllm_latent_norm_store(void* out, const void* in, int64_t in_row_stride, const float* weight, float eps, void* cache,
                            int64_t num_slots, const int64_t* slots, int64_t rows, int rank, int padded, int dtype,
                            void* stream);
int mvllm_head_linear(void* out, int64_t out_row_stride, int64_t out_head_stride, const void* x, int64_t x_row_stride,
                      int64_t x_head_stride, const void* w, int64_t rows, int num_heads, int N, int K, int dtype,
                      void* stream);
size_t mvllm_latent_decode_workspace_bytes(int rows, int num_heads, int padded, int64_t max_keys, int dtype);
int mvllm_latent_decode(void* out, const void* q, const void* cache, const int32_t* block_tables, int table_width,
                        const int32_t* row_entry, const int64_t* lens, int rows, int num_heads, int padded, int block_size,
                        int64_t num_blocks, float scale, int dtype, void* workspace, size_t workspace_bytes, void* stream);

/*
 * Mixture of experts (csrc/moe.hip).
 * mvllm_moe_route: ids int32 [rows, top], weights fp32 [rows, top] from fp32 logits: s = sigmoid(z), choice = s + correction
 *   (fp32 [experts] or NULL); with groups > 1 only experts of the `keep` groups of neighbours with the largest sums of their
 *   two largest choices are open; weights = s / (sum + 1e-20).
 * mvllm_moe_plan: (token, choice) pairs sorted by expert, into `plan` (mvllm_moe_plan_bytes; its first `pairs` int32 are the
 *   sorted place of every pair).
 * mvllm_moe_linear: w [experts, N, K]; glu: gate and up rows in turns of 32, result silu(gate) * up.  With a plan: row p of
 *   out is sorted place p, reading x row pair / per_token (per_token > 0) or row p.  Without (bf16, at most 512 pairs, meant
 *   for a few): row p of out is pair p, reading x row p / per_token or row p.  K % 64 == 0,
 *   N % 16 == 0 (glu: 64), bf16 and fp32.
 */
int mvllm_moe_route(int32_t* ids, float* weights, const float* logits, int64_t logit_row_stride, const float* correction,
                    int64_t rows, int experts, int top, int groups, int keep, void* stream);
size_t mvllm_moe_plan_bytes(int64_t pairs, int experts);
int mvllm_moe_plan(void* plan, size_t plan_bytes, const int32_t* ids, int64_t pairs, int experts, void* stream);
int mvllm_moe_linear(void* out, int64_t out_row_stride, const void* x, int64_t x_row_stride, const void* w,
                     const int32_t* ids, void* plan, int64_t pairs, int experts, int N, int K, int per_token, int glu,
                     int dtype, void* stream);

/*
 * ... and for models whose router is a softmax and whose experts have a clamped gate:
 * mvllm_moe_route_softmax: s = softmax(z) over experts + identity outputs, choice = s + correction, weights = s (renormalize:
 *   s / (sum + 1e-20)).  The last `identity` outputs stand for no expert: their id is -1, and the plan leaves such pairs out
 *   (their place is -1, their rows of the products are not written).
 * mvllm_moe_linear_clamped: mvllm_moe_linear with g' sigmoid(alpha g') (u' + shift) behind it, g' = min(g, limit), u' = u clamped
 *   to +-limit.
 * mvllm_gated_unit: the same of dense rows: in [rows, in_row_stride] = g [width] | u [width], out [rows, out_row_stride].
 * mvllm_stream_norm_identity: mvllm_stream_norm whose choices with ids < 0 (int32 [rows, top]) read row t of `self`
 *   [rows, self_row_stride] instead of a row of parts.
 */
int mvllm_moe_route_softmax(int32_t* ids, float* weights, const float* logits, int64_t logit_row_stride,
                            const float* correction, int64_t rows, int experts, int identity, int top, int renormalize,
                            void* stream);
int mvllm_moe_linear_clamped(void* out, int64_t out_row_stride, const void* x, int64_t x_row_stride, const void* w,
                             const int32_t* ids, void* plan, int64_t pairs, int experts, int N, int K, int per_token,
                             float alpha, float limit, float shift, int dtype, void* stream);
int mvllm_gated_unit(void* out, int64_t out_row_stride, const void* in, int64_t in_row_stride, int64_t rows, int width,
                     float alpha, float limit, float shift, int dtype, void* stream);
int mvllm_stream_norm_identity(void* out, int64_t out_row_stride, float* x_out, const float* x, const void* y,
                               int64_t y_row_stride, const void* parts, int64_t part_row_stride, const int32_t* part_row,
                               const float* weights, int top, const int32_t* ids, const void* self,
                               int64_t self_row_stride, const float* gate, int64_t gate_row_stride, const float* scale,
                               const float* hc_out, const float* hc_mix, const float* hc_in, const float* gain, float eps,
                               int64_t rows, int streams, int width, int dtype, void* stream);

/*
 * Windowed attention over rows that are keys and values at once, or over keys in two parts with values of their own
 * (csrc/window_prefill.hip, csrc/window_decode.hip).  A query sees the `window` keys up to its own (0: all of them);
 *     score = scale * t(p) * q . k - slopes[h] * distance,   t(p) = 1 + temp_coef ln(floor((p + 1) / temp_every) + 1)
 * (slopes fp32 [H] or NULL; temp_every 0: t = 1), out = softmax . v, times sigmoid(gate) where gate is not NULL (head h's
 * columns at h * gate_head_stride; stride 1: one number for all of a head's columns).  Strides are in elements; bf16 and fp32.
 * mvllm_window_prefill: entries of packed queries (cu_q) over packed keys (cu_k); query i of an entry stands at key
 *   (keys - queries) + i.  q: head h at h * q_head_stride, [dim | rot]; k: kv head g at g * k_head_stride, [dim]; k2 [rot], shared
 *   by all heads, or NULL with rot 0; v like k, or NULL: the values are the keys.  positions int64 [total_q] (t only).  Tiled in
 *   bf16 for dim 32, 64, 96, 128, 192, 256: without v, with v alone (no slopes), and with v and k2 for rot 32 and 64 (no slopes);
 *   else dim and rot up to 512.
 * mvllm_window_decode: single query rows over a paged cache [num_blocks, block_size, kv heads, padded] (padded a multiple of 32)
 *   whose rows are keys and, their first `values` columns (padded, or 512 of 576), values.  lens int64 [rows]: position + 1;
 *   ring > 0: token p lies at place p mod ring of its entry's table (ring >= window + the most rows an entry has in a call - 1),
 *   0: at place p.  Everything else as for mvllm_latent_decode.
 * mvllm_window_decode_split: the same over rows of `keys` columns of a key and behind them `values` of its value (multiples of 32;
 *   tiled in bf16 where both are one of the widths of the tiled prefill).  Workspace: mvllm_window_decode_workspace_bytes with
 *   padded = keys + values.
 * mvllm_latent_rope_store: mvllm_latent_norm_store with a part behind the latent, columns rot_col .. rot_col + rot of a row, that is
 *   not normed; its first rot_dims columns turn by rot_table fp32 [max_position, rot_dims / 2, 2] (cos, sin) in pairs (2i, 2i + 1) if
 *   interleaved, else (i, i + rot_dims / 2).  out_rows int64 [rows] (< 0: none) or NULL: rows of `out`.  in2 != NULL: a second plain
 *   norm in the same launch, out2 [rows, padded2] = rms(in2[:rank2]) * weight2.
 * mvllm_head_rope: the same rotation of columns x_col .. x_col + rot of every head of x, in place; the first `first_rows` rows go to
 *   columns out_col .. out_col + out_width of first_out instead, zeros behind the part.
 * mvllm_copy_rows: row src_rows[t] of src to row dst_rows[t] of dst and dst2_rows[t] of dst2 (indices int64, negative ones are
 *   skipped, NULL: row t; dst or dst2 NULL: none); rows a multiple of 16 bytes.
 */
int mvllm_window_prefill(void* out, int64_t out_row_stride, int64_t out_head_stride, const void* q, int64_t q_row_stride,
                         int64_t q_head_stride, const void* k, int64_t k_row_stride, int64_t k_head_stride, const void* k2,
                         int64_t k2_row_stride, const void* v, int64_t v_row_stride, int64_t v_head_stride, const void* gate,
                         int64_t gate_row_stride, int64_t gate_head_stride, const int32_t* cu_q, const int32_t* cu_k,
                         const int64_t* positions, const float* slopes, int num_seqs, int64_t total_q, int num_heads,
                         int num_kv_heads, int dim, int rot, int window, float scale, float temp_coef, float temp_every,
                         int dtype, void* stream);
size_t mvllm_window_decode_workspace_bytes(int rows, int num_heads, int num_kv_heads, int padded, int values, int64_t max_keys,
                                           int dtype);
int mvllm_window_decode(void* out, int64_t out_row_stride, int64_t out_head_stride, const void* q, int64_t q_row_stride,
                        int64_t q_head_stride, const void* cache, const int32_t* block_tables, int table_width,
                        const int32_t* row_entry, const int64_t* lens, const float* slopes, const void* gate,
                        int64_t gate_row_stride, int64_t gate_head_stride, int rows, int num_heads, int num_kv_heads,
                        int padded, int values, int block_size, int64_t num_blocks, int window, int ring, float scale,
                        float temp_coef, float temp_every, int dtype, void* workspace, size_t workspace_bytes, void* stream);
int mvllm_window_decode_split(void* out, int64_t out_row_stride, int64_t out_head_stride, const void* q, int64_t q_row_stride,
                              int64_t q_head_stride, const void* cache, const int32_t* block_tables, int table_width,
                              const int32_t* row_entry, const int64_t* lens, const float* slopes, const void* gate,
                              int64_t gate_row_stride, int64_t gate_head_stride, int rows, int num_heads, int num_kv_heads,
                              int keys, int values, int block_size, int64_t num_blocks, int window, int ring, float scale,
                              float temp_coef, float temp_every, int dtype, void* workspace, size_t workspace_bytes, void* stream);
int mvllm_latent_rope_store(void* out, const int64_t* out_rows, const void* in, int64_t in_row_stride, const float* weight,
                            float eps, const float* rot_table, int rot_col, int rot, int rot_dims, int interleaved,
                            int64_t max_position, const int64_t* positions, void* cache, int64_t num_slots,
                            const int64_t* slots, void* out2, const void* in2, int64_t in2_row_stride, const float* weight2,
                            int rank2, int padded2, int64_t rows, int rank, int padded, int dtype, void* stream);
int mvllm_head_rope(void* x, int64_t x_row_stride, int64_t x_head_stride, int x_col, void* first_out, int64_t out_row_stride,
                    int64_t out_head_stride, int out_col, int out_width, int64_t first_rows, const float* table, int rot,
                    int rot_dims, int interleaved, int64_t max_position, const int64_t* positions, int64_t rows, int num_heads,
                    int dtype, void* stream);
int mvllm_copy_rows(void* dst, int64_t dst_row_stride, int64_t dst_count, const int64_t* dst_rows, void* dst2,
                    int64_t dst2_row_stride, int64_t dst2_count, const int64_t* dst2_rows, const void* src,
                    int64_t src_row_stride, int64_t src_count, const int64_t* src_rows, int64_t rows, int width, int dtype,
                    void* stream);

/*
 * out = gelu(in), z / 2 (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3))); rows of `width` numbers (a multiple of 16 bytes), strides in
 * elements.  mvllm_linear_small_m_gelu: mvllm_linear_small_m with it behind the bias, rounded once.
 */
int mvllm_gelu_tanh(void* out, int64_t out_row_stride, const void* in, int64_t in_row_stride, int64_t rows, int width, int dtype,
                    void* stream);
int mvllm_linear_small_m_gelu(void* out, const void* x, const void* w, const void* bias, int64_t x_row_stride, int M, int N, int K,
                              int dtype, void* stream);

/*
 * Between the sublayers of a decoder that norms what they return (csrc/post_norm.hip): x_out = x + norm(y) * gain (fp32
 * [rows, width]; may be x itself, or NULL), out = x_out, or norm(x_out) * final_gain where that is not NULL, in dtype, zeros from
 * `width` to out_row_stride.  norm divides by sqrt(mean of squares + eps), with `centred` after taking the mean off.
 * mvllm_embed_rows: x_out = embed[token] * scale, out = x_out.
 */
int mvllm_post_norm(void* out, int64_t out_row_stride, float* x_out, const float* x, const void* y, int64_t y_row_stride,
                    const float* gain, const float* final_gain, float eps, int centred, int64_t rows, int width, int dtype,
                    void* stream);
int mvllm_embed_rows(void* out, int64_t out_row_stride, float* x_out, const void* embed, int64_t vocab, float scale,
                     const int64_t* tokens, int64_t rows, int width, int dtype, void* stream);

/*
 * Attention whose heads' scores are mixed before the softmax (csrc/talk.h): s_h = sum_g talk[h, g] q_g . k, with an optional sink
 * per head (one more exp(sink) in the denominator).  Queries carry the score scale and log2 e: scores are exponents of two as
 * they come.  q [rows, H, dim] contiguous, talk fp32 [H, H], sinks fp32 [H] or NULL, out: head h at h * out_head_stride.
 * mvllm_talk_prefill: pieces of packed queries (cu_q); keys and values [*, Hkv, dim], packed (cu_k: more keys than queries in front,
 *   NULL: as many) or, with block_tables, a paged cache [num_blocks, block_size, Hkv, dim].  out_rows int32 [total_q] or NULL: rows
 *   of out.
 * mvllm_talk_decode: single rows over the cache, lens int64 [rows] keys each, a table per row; the workspace holds partial results.
 * bf16 and fp32; H up to 64, H * dim up to 16384.  Tiled in bf16 for dim 32, 64, 96, 128 and up to 8 kv heads (prefill: up to 8
 * groups of four heads that share one, and talk rounded to bf16).
 */
int mvllm_talk_prefill(void* out, int64_t out_row_stride, int64_t out_head_stride, const int32_t* out_rows, const void* q,
                       const void* k, const void* v, const int32_t* cu_q, const int32_t* cu_k, const int32_t* block_tables,
                       int table_width, int block_size, int64_t num_blocks, const float* talk, const float* sinks, int num_seqs,
                       int64_t total_q, int num_heads, int num_kv_heads, int dim, int dtype, void* stream);
size_t mvllm_talk_decode_workspace_bytes(int rows, int num_heads, int num_kv_heads, int dim, int64_t max_keys, int dtype);
int mvllm_talk_decode(void* out, int64_t out_row_stride, int64_t out_head_stride, const void* q, const void* k_cache,
                      const void* v_cache, const int32_t* block_tables, int table_width, const int64_t* lens, const float* talk,
                      const float* sinks, int rows, int num_heads, int num_kv_heads, int dim, int block_size, int64_t num_blocks,
                      int dtype, void* workspace, size_t workspace_bytes, void* stream);

#ifdef __cplusplus
}
#endif
#endif /* MINIVLLM_AMD_H_ */
