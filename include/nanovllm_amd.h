/*
 * nanovllm_amd -- C ABI of the MI355X (gfx950) attention hot path for nano-vllm.
 *
 * Every entry point borrows raw device pointers for the duration of one asynchronous
 * launch on the HIP stream it is given.  The library never allocates or frees device
 * memory, never synchronises and never reads device data on the host, so all calls are
 * legal under stream capture.  Scratch memory is supplied by the caller (query its size
 * with the *_workspace_bytes functions).  Arguments are validated on the host before any
 * launch; a non-zero return means nothing was enqueued.
 *
 * Dtypes / geometry: bf16 tensors, int32 index tensors, head_dim 128, KV blocks of 256, 512,
 * 1024, 2048 or 4096 tokens, num_heads / num_kv_heads from 1 to 8 (decode; prefill takes any
 * multiple).  Anything else is rejected with
 * NVA_ERR_UNSUPPORTED_GEOMETRY rather than served by a slow path.
 *
 * File:line citations name the reference (nano-vllm) interface each entry point replaces.
 */
#ifndef NANOVLLM_AMD_H
#define NANOVLLM_AMD_H

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

enum nva_status {
    NVA_OK = 0,
    NVA_ERR_NULL_POINTER = 1,         /* a required pointer is NULL                         */
    NVA_ERR_BAD_SHAPE = 2,            /* negative / inconsistent counts                     */
    NVA_ERR_UNSUPPORTED_GEOMETRY = 3, /* head_dim, block_size or GQA group not built        */
    NVA_ERR_BAD_STRIDE = 4,           /* row stride smaller than a row, or not 16-byte      */
    NVA_ERR_MISALIGNED = 5,           /* base pointer not 16-byte aligned                   */
    NVA_ERR_WORKSPACE_TOO_SMALL = 6,  /* workspace_bytes below *_workspace_bytes()          */
    NVA_ERR_LAUNCH_FAILED = 7,        /* hipGetLastError() after the launch was not success */
    NVA_ERR_NO_DEVICE = 8,            /* no HIP device visible                              */
    NVA_ERR_SCRATCH_TOO_SMALL = 9     /* problem exceeds the library's built-in scratch array */
};

/* Element type of the entry points that take bf16 or fp32 tensors. */
enum nva_dtype { NVA_DTYPE_BF16 = 0, NVA_DTYPE_F32 = 1 };

/* which keys the query at position p sees: [p / span * span, p], or the last `span` up to and with p */
enum nva_mask { NVA_MASK_CHUNKS = 0, NVA_MASK_WINDOW = 1 };

/* norms of nva_qkv_prepare: over a whole projection instead of every head; q and k normed without a weight where theirs is
 * NULL; every head's values normed, without a weight */
enum nva_qkv_norms { NVA_QKV_NORM_WHOLE = 1, NVA_QKV_NORM_UNIT = 2, NVA_QKV_NORM_VALUES = 4 };

/* weights of nva_router: softmax over all experts, normalised over the chosen ones, or the chosen logits' sigmoids as they are */
enum nva_score { NVA_SCORE_SOFTMAX = 0, NVA_SCORE_SIGMOID = 1 };

/* Library version, (major << 16) | minor. */
int nva_version(void);

/* Static, human-readable name of a status code (never NULL). */
const char *nva_status_string(int status);

/* Number of visible HIP devices; NVA_ERR_NO_DEVICE (and *count = 0) when there is none. */
int nva_device_count(int *count);

/*
 * KV-cache slot scatter.  Replaces store_kvcache / store_kvcache_kernel
 * (nanovllm/layers/attention.py:10-40).
 *
 * key/value: bf16 [n_tokens, num_kv_heads, head_dim], innermost two dims dense, row
 * strides in ELEMENTS (value is a strided view of the fused qkv buffer in the model).
 * k_cache/v_cache: bf16, addressed flat as [num_slots, num_kv_heads*head_dim].
 * slot_mapping: int32 [n_tokens]; row i goes to cache row slot_mapping[i]; -1 skips the
 * row.  Slots outside [0, num_slots) are skipped as well instead of written out of
 * bounds.  Duplicate slots are safe; which row wins is unspecified (as in the reference).
 * The copy is bit-exact.  n_tokens == 0 is a no-op.
 */
int nva_store_kvcache(const void *key, int64_t key_row_stride,
                      const void *value, int64_t value_row_stride,
                      void *k_cache, void *v_cache,
                      const int32_t *slot_mapping,
                      int32_t n_tokens, int32_t num_kv_heads, int32_t head_dim,
                      int64_t num_slots, void *stream);

/*
 * Paged single-query (decode) attention.  Replaces the flash_attn_with_kvcache call of
 * Attention.forward (nanovllm/layers/attention.py:71-74).
 *
 * q: bf16 [batch, num_heads, head_dim], row stride q_row_stride elements, heads dense.
 * k_cache/v_cache: bf16 [num_blocks, block_size, num_kv_heads, head_dim], dense.
 * block_tables: int32 [batch, max_blocks] with row stride bt_row_stride; only entries
 * j < ceil(context_lens[b] / block_size) are dereferenced (the rest may be -1 or stale);
 * an entry outside [0, num_blocks) contributes nothing instead of faulting.
 * context_lens: int32 [batch]; 0 yields an all-zero output row.
 * out: bf16 [batch, num_heads, head_dim] dense (the reference's [B,1,Hq,Dh]).
 * workspace: at least nva_paged_decode_workspace_bytes() bytes, 16-byte aligned; holds
 * split partials, contents need no initialisation.  Calls that overlap in time need
 * separate workspaces; calls ordered on one stream (every layer of a model) can share one.
 * Launch geometry depends only on (batch, heads), never on device data, so a call can be
 * captured in a HIP graph and replayed with new contents.
 */
size_t nva_paged_decode_workspace_bytes(int32_t batch, int32_t num_heads, int32_t head_dim,
                                        int32_t max_blocks);

int nva_paged_decode_attn(const void *q, int64_t q_row_stride,
                          const void *k_cache, const void *v_cache,
                          const int32_t *block_tables, int32_t bt_row_stride, int32_t max_blocks,
                          const int32_t *context_lens,
                          void *out, void *workspace, size_t workspace_bytes,
                          int32_t batch, int32_t num_heads, int32_t num_kv_heads,
                          int32_t head_dim, int32_t block_size, int32_t num_blocks,
                          float scale, void *stream);

/*
 * The same operation for a caller that makes several calls over the SAME context_lens and
 * block_tables contents, batch, head counts and workspace, ordered on one stream -- the
 * layers of one decode step (the loop over decoder layers around
 * nanovllm/layers/attention.py:71-74 changes only q and the cache pointers).
 *   plan == NVA_PLAN_BUILD: as nva_paged_decode_attn; the work split it derives from
 *     context_lens and block_tables stays in the workspace.
 *   plan == NVA_PLAN_REUSE: takes the split the last NVA_PLAN_BUILD call left in this
 *     workspace instead of deriving it again (saves a few microseconds per launch).  The caller
 *     guarantees that call had the same batch, head counts, num_blocks and table contents
 *     and that nothing else wrote the workspace since; otherwise the result is undefined
 *     (memory accesses stay inside the caches as long as the old block numbers were valid).
 * Batches above 1024 sequences are run as several launches and always rebuild.
 */
enum { NVA_PLAN_BUILD = 0, NVA_PLAN_REUSE = 1 };

int nva_paged_decode_attn_planned(const void *q, int64_t q_row_stride,
                                  const void *k_cache, const void *v_cache,
                                  const int32_t *block_tables, int32_t bt_row_stride,
                                  int32_t max_blocks, const int32_t *context_lens,
                                  void *out, void *workspace, size_t workspace_bytes,
                                  int32_t batch, int32_t num_heads, int32_t num_kv_heads,
                                  int32_t head_dim, int32_t block_size, int32_t num_blocks,
                                  float scale, int32_t plan, void *stream);

/*
 * Causal variable-length prefill attention, optionally reading K/V through the paged
 * cache.  Replaces the flash_attn_varlen_func call of Attention.forward
 * (nanovllm/layers/attention.py:64-70).
 *
 * q: bf16 [total_q, num_heads, head_dim], row stride q_row_stride elements.
 * block_tables == NULL: k/v are packed bf16 [total_k, num_kv_heads, head_dim] with their
 *   own row strides, sequence b owning rows cu_seqlens_k[b]..cu_seqlens_k[b+1].
 * block_tables != NULL: k/v are ignored (may be NULL) and every sequence reads its
 *   cu_seqlens_k[b+1]-cu_seqlens_k[b] logical positions from k_cache/v_cache through
 *   block_tables[b] (int32 [batch, max_blocks], row stride bt_row_stride, -1 padded).
 *   A table entry outside [0, num_blocks) that a sequence's keys reach contributes nothing
 *   (its 256 keys drop out) instead of faulting.
 * The causal mask is aligned to the END of the keys: query i of a sequence sees keys
 * j <= i + (Lk - Lq).  Empty query spans are no-ops.
 * out: bf16 [total_q, num_heads, head_dim] dense.  max_seqlen_q bounds the launch grid.
 */
int nva_varlen_prefill_attn(const void *q, int64_t q_row_stride,
                            const void *k, int64_t k_row_stride,
                            const void *v, int64_t v_row_stride,
                            const void *k_cache, const void *v_cache,
                            const int32_t *block_tables, int32_t bt_row_stride, int32_t max_blocks,
                            const int32_t *cu_seqlens_q, const int32_t *cu_seqlens_k,
                            int32_t batch, int32_t max_seqlen_q, int32_t max_seqlen_k,
                            void *out,
                            int32_t num_heads, int32_t num_kv_heads, int32_t head_dim,
                            int32_t block_size, int32_t num_blocks,
                            float scale, void *stream);

/*
 * Temperature / exponential-race sampler.  Replaces Sampler.forward
 * (nanovllm/layers/sampler.py:10-15):
 *     token[b] = argmax_i softmax(float(logits[b]) / T[b])[i] / max(E[b,i], 1e-10)
 * with the first index winning ties.
 *
 * logits: bf16 [batch, vocab], row stride logits_row_stride elements.
 * temperatures: fp32 [batch].  T == 0 selects greedy argmax(logits) for that row (an
 * extension; the reference forbids T <= 1e-10, nanovllm/sampling_params.py:11).
 * noise: fp32 [batch, vocab] Exp(1) draws (row stride noise_row_stride): the formula above is
 * evaluated (scores relative to the maximum of each 4096-column chunk, rescaled to the row) and a
 * draw can be replayed; the argmax differs from the formula only between scores that agree to fp32
 * rounding.  NULL: the token is drawn from the same categorical distribution softmax(logits / T) by a
 * tree of inverse-CDF steps (row -> chunk of 8192 columns -> one of 4 column groups -> one of its 64
 * lanes -> one of the lane's 32 columns; at every level the first branch whose running sum of
 * weights exceeds u * total), each level with its own 32-bit uniform from Philox4x32-10 keyed by
 * (seed, offset, row, chunk); the same (seed, offset) reproduces the draw.  Sums are fp32 and a
 * conditional probability below 2^-32 at a level is not resolved.
 * out_tokens: int64 [batch].
 * workspace: at least nva_sample_workspace_bytes() bytes, 16-byte aligned.  Its size (and the limit
 * of nva_sample_static below) is counted in records of 2048 columns, the finest chunking any path
 * has used; the present chunkings (4096 columns with a noise tensor, 8192 without) need fewer.
 */
size_t nva_sample_workspace_bytes(int32_t batch, int32_t vocab);

int nva_sample(const void *logits, int64_t logits_row_stride,
               const float *temperatures,
               const float *noise, int64_t noise_row_stride,
               uint64_t seed, uint64_t offset,
               int64_t *out_tokens,
               void *workspace, size_t workspace_bytes,
               int32_t batch, int32_t vocab, void *stream);

/*
 * nva_sample without a workspace argument, for callers that cannot allocate device memory (code
 * under HIP graph capture, tight serving loops, harnesses that forbid hipMalloc).  It has no
 * counterpart in the reference.  Same arguments, kernels and results as nva_sample; the per-chunk
 * records live in a device array built into the library (2 MiB per GPU the library is used on, held
 * until the process ends), which bounds the problem size:
 *     batch * ceil(vocab / 2048) <= NVA_SAMPLE_STATIC_MAX_RECORDS      (1747 rows at vocab 151,936)
 * Larger problems return NVA_ERR_SCRATCH_TOO_SMALL and launch nothing.  The call allocates and frees
 * nothing; the first call on a device looks the array's address up (make that call outside stream
 * capture).  All calls on one GPU share the array: calls that overlap in time on one GPU race and
 * must be ordered by the caller (one stream, or events); nothing needs clearing between calls.
 */
#define NVA_SAMPLE_STATIC_MAX_RECORDS 131072

int nva_sample_static(const void *logits, int64_t logits_row_stride,
                      const float *temperatures,
                      const float *noise, int64_t noise_row_stride,
                      uint64_t seed, uint64_t offset,
                      int64_t *out_tokens,
                      int32_t batch, int32_t vocab, void *stream);

/*
 * ---- steps either side of the hot path (the callers' element-wise glue) ----------------
 */

/*
 * RMSNorm, optionally fused with the residual add.  Replaces RMSNorm.rms_forward /
 * add_rms_forward (nanovllm/layers/layernorm.py:16-40).
 *   residual == NULL: out = bf16(x * rsqrt(mean(x^2) + eps)) * weight
 *   otherwise:        s = x + residual (fp32); residual_out = bf16(s);
 *                     out = bf16(s * rsqrt(mean(s^2) + eps)) * weight
 * x / residual: bf16 [rows, hidden] with row strides in elements; weight bf16 [hidden];
 * out / residual_out: bf16 [rows, hidden] dense.  hidden % 8 == 0, hidden <= 4096.
 */
int nva_rms_norm(const void *x, int64_t x_row_stride,
                 const void *residual, int64_t residual_row_stride,
                 const void *weight, void *out, void *residual_out,
                 int32_t rows, int32_t hidden, float eps, void *stream);

/*
 * Final norm of a prefill step on the rows that feed the LM head only.  Replaces the pair
 * "hidden_states, _ = self.norm(hidden_states, residual)" (nanovllm/models/qwen3.py:176) +
 * "x = x[cu_seqlens_q[1:] - 1].contiguous()" (nanovllm/layers/embed_head.py:56-61): the reference
 * normalises all total_rows rows and then copies the last row of every sequence; this reads and
 * normalises those batch rows alone, bit-identical to the rows nva_rms_norm would have produced.
 *   i = cu_seqlens_q[b + 1] - 1  (a negative index wraps to total_rows + i, as torch indexing does;
 *                                 an empty query span picks the previous sequence's last row, as in
 *                                 the reference; indices are clamped to the tensor)
 *   out[b] = bf16(s * rsqrt(mean(s^2) + eps)) * weight,  s = x[i] (+ residual[i] when residual != NULL)
 * x / residual: bf16 [total_rows, hidden], row strides in elements; cu_seqlens_q: int32 [batch + 1];
 * out: bf16 [batch, hidden] dense.  hidden % 8 == 0, hidden <= 4096.
 */
int nva_gather_last_rms_norm(const void *x, int64_t x_row_stride,
                             const void *residual, int64_t residual_row_stride,
                             const int32_t *cu_seqlens_q, const void *weight, void *out,
                             int32_t batch, int32_t total_rows, int32_t hidden, float eps, void *stream);

/*
 * Per-head RMSNorm of q and k followed by the neox rotary embedding, optionally fused with the
 * KV-cache scatter.  Replaces the q_norm / k_norm / rotary_emb sequence of
 * Qwen3Attention.forward (nanovllm/models/qwen3.py:76-79; nanovllm/layers/rotary_embedding.py:6-48)
 * and, when a cache is given, the store_kvcache call of Attention.forward
 * (nanovllm/layers/attention.py:62-63) for the same rows.
 * qkv: bf16 [n_tokens, (num_heads + 2*num_kv_heads) * head_dim], row stride in elements
 * (q heads, then k heads, then v heads).  positions: int64 [n_tokens].
 * q_weight / k_weight: bf16 [head_dim].  rope_cache: fp32 [max_position, head_dim], cos in
 * the first half of a row, sin in the second; positions are clamped to [0, max_position).
 * q_out: bf16 [n_tokens, num_heads, head_dim], k_out: bf16 [n_tokens, num_kv_heads, head_dim],
 * both dense.  head_dim must be 128.
 * k_cache / v_cache / slot_mapping: all NULL (no scatter), or the flat caches
 * [num_slots, num_kv_heads * head_dim] and int32 [n_tokens] slots: the rotated key row and the
 * (unchanged) value row of token i are also written to cache row slot_mapping[i], bit-identical
 * to what nva_store_kvcache would write from k_out and the v view; -1 / out-of-range skips.
 * Every tensor pointer must be 16-byte aligned and qkv_row_stride a multiple of 8 elements
 * (NVA_ERR_MISALIGNED / NVA_ERR_BAD_STRIDE otherwise): all accesses are 16 bytes per lane.
 */
int nva_qk_norm_rope(const void *qkv, int64_t qkv_row_stride, const int64_t *positions,
                     const void *q_weight, const void *k_weight, const float *rope_cache,
                     int32_t max_position, void *q_out, void *k_out,
                     void *k_cache, void *v_cache, const int32_t *slot_mapping, int64_t num_slots,
                     int32_t n_tokens, int32_t num_heads, int32_t num_kv_heads, int32_t head_dim,
                     float eps, void *stream);

/*
 * SwiGLU gate.  Replaces SiluAndMul.forward (nanovllm/layers/activation.py:11-14):
 * out[r, i] = bf16(silu(x[r, i])) * x[r, inter + i].
 * x: bf16 [rows, 2*inter] (row stride in elements), out: bf16 [rows, inter] dense, inter % 8 == 0.
 */
int nva_silu_and_mul(const void *x, int64_t x_row_stride, void *out,
                     int32_t rows, int32_t inter, void *stream);

/*
 * Brings the per-step decode inputs from a pinned host buffer into their device buffer with one
 * kernel (the device reads host memory directly; no copy engine, no second launch), and feeds the
 * tokens sampled by the previous step to this one without a trip through the host.  It stands
 * where the reference copies input_ids, positions, slot_mapping, context_lens and block_tables
 * from the host one by one (nanovllm/engine/model_runner.py:162-179,197-203).
 *   dst[0 .. nbytes) = src_host[0 .. nbytes)                        (nbytes % 16 == 0, both 16-byte aligned)
 *   then, with ids = (int64*)(dst + ids_offset) and idx = (int32*)(src_host + index_offset), for i < n:
 *   ids[i] = prev_tokens[idx[i]] where 0 <= idx[i] < n_prev         (other rows keep the host's value)
 * src_host must be device-accessible host memory (hipHostMalloc / a pinned torch tensor).
 * prev_tokens: int64 [n_prev], the sampler's output of the previous step; NULL with n_prev == 0.
 */
int nva_stage_decode_inputs(void *dst, const void *src_host, int64_t nbytes, int64_t ids_offset,
                            int64_t index_offset, int32_t n, const int64_t *prev_tokens, int32_t n_prev,
                            void *stream);

/*
 * ---- layered models: mixers and the steps around them -----------------------------------
 * bf16 or fp32 tensors (dtype: enum nva_dtype), fp32 residual stream, no counterpart in the reference.
 * A step's rows are either portions of sequences (cu_seqlens_q [n_seqs + 1]: row bounds; seq_lens: tokens
 * of each sequence once these rows are in; token_seq [n_tokens]: sequence of every row) or single tokens
 * (cu_seqlens_q NULL: row i is the newest token of sequence i, at position seq_lens[i] - 1; a row with
 * seq_lens[i] <= 0 is padding: its result is zero and nothing is stored).  Recurrent state and carried
 * rows live in slots; a sequence whose rows begin at position 0 starts from zeros whatever its slot
 * holds, and slots outside [0, num_state_slots) are neither read nor written.  Sizes that are multiples
 * of 8 with 16-byte aligned tensors take the vector paths; any other size runs too.
 */

/* residual[r] = table[ids[r]] * scale (fp32); out[r] = layer_norm(residual[r]) * weight + bias.
 * ids are clamped to [0, vocab).  Variance is the mean of the squared deviations, eps inside the root. */
int nva_embed_norm(const int64_t *ids, const void *table, float scale, const void *weight, const void *bias,
                   float *residual, void *out, int32_t rows, int32_t width, int32_t vocab, float eps,
                   int32_t dtype, void *stream);

/* residual[r] += layer_norm(y[r]) * post_weight + post_bias, in place, fp32;
 * out[r] = layer_norm(residual[r]) * next_weight + next_bias.
 * rows_of (int32 [rows], may be NULL): out[r] is computed from row rows_of[r] of y and residual
 * (clamped to [0, src_rows)) and residual is not written; without it rows == src_rows. */
int nva_post_add_norm(const void *y, int64_t y_row_stride, float *residual, const void *post_weight,
                      const void *post_bias, const void *next_weight, const void *next_bias, void *out,
                      const int32_t *rows_of, int32_t rows, int32_t src_rows, int32_t width, float eps,
                      int32_t dtype, void *stream);

/* x: [rows, 2 * inter] (gate | up, row stride in elements).  g = min(gate, limit), u = clamp(up, -limit, limit),
 * out = g * sigmoid(alpha * (g + cubic * g^3)) * (u + shift).  (limit infinity, alpha 2 sqrt(2 / pi), cubic 0.044715, shift 0: the
 * tanh form of gelu(gate), times up.) */
int nva_clamped_gate(const void *x, int64_t x_row_stride, void *out, int32_t rows, int32_t inter, float limit,
                     float alpha, float cubic, float shift, int32_t dtype, void *stream);

/* out = max(x, 0)^2; x: [rows, width] (row stride in elements), out dense, may be x. */
int nva_squared_relu(const void *x, int64_t x_row_stride, void *out, int32_t rows, int32_t width, int32_t dtype,
                     void *stream);

/* x = cap * tanh(x / cap), in place; x: [rows, width] dense. */
int nva_soft_cap(void *x, int32_t rows, int32_t width, float cap, int32_t dtype, void *stream);

/* q, k and v of an attention layer: causal convolution over time on every channel, rotary embedding of
 * the first rot_dims elements of each q and k head (pairs i, i + rot_dims / 2), q to q_out, k and v to
 * their cache slots.
 * qkv: [n_tokens, channels], channels = (num_heads + num_kv_heads) * qk_dim + num_kv_heads * v_dim.
 * conv_weight: [taps, channels], tap taps - 1 meets the row itself; 1 <= taps <= 16.
 * conv_state: [num_state_slots, taps - 1, channels], the last projected rows of every sequence, oldest
 * first; read for rows before a portion, updated by the call.
 * rope_cache: fp32 [max_position, rot_dims], cos in the first half of a row, sin in the second. */
int nva_conv_rope_store(const void *qkv, int64_t qkv_row_stride, const void *conv_weight, void *conv_state,
                        const int32_t *state_slots_of_seq, const int32_t *cu_seqlens_q, const int32_t *seq_lens,
                        const int32_t *token_seq, const float *rope_cache,
                        void *q_out, void *k_cache, void *v_cache, const int32_t *slot_mapping,
                        int64_t num_slots, int32_t n_tokens, int32_t n_seqs, int32_t num_heads,
                        int32_t num_kv_heads, int32_t qk_dim, int32_t v_dim, int32_t rot_dims, int32_t taps,
                        int32_t max_position, int32_t num_state_slots, int32_t dtype, void *stream);

/* Softmax attention inside position chunks: the query at position p sees keys [p / chunk * chunk, p] of
 * its sequence, all of them read from the paged cache (this step's rows must be stored already).
 * score = (q . k) * scale, then softcap * tanh(score / softcap) where softcap > 0.
 * q: [n_tokens, num_heads, qk_dim] (row stride in elements), caches [num_blocks, block_size, num_kv_heads,
 * qk_dim or v_dim], block_tables int32 [n_seqs, >= max_blocks]; out: [n_tokens, num_heads, v_dim] dense.
 * A key behind a table entry outside [0, num_blocks) is not seen.
 * workspace: partial results of single-token rows, nva_chunk_attn_workspace_bytes() bytes, 16-byte aligned
 * (NULL where that is 0, and for portions); needs no initialisation.  max_seqlen_q: longest portion. */
size_t nva_chunk_attn_workspace_bytes(int32_t n_tokens, int32_t num_heads, int32_t num_kv_heads, int32_t v_dim,
                                      int32_t max_blocks, int32_t block_size, int32_t chunk);
int nva_chunk_attn(const void *q, int64_t q_row_stride, const void *k_cache, const void *v_cache,
                   const int32_t *block_tables, int64_t bt_row_stride, int32_t max_blocks,
                   const int32_t *cu_seqlens_q, const int32_t *seq_lens, const int32_t *token_seq, void *out,
                   void *workspace, size_t workspace_bytes,
                   int32_t n_tokens, int32_t n_seqs, int32_t max_seqlen_q, int32_t num_heads,
                   int32_t num_kv_heads, int32_t qk_dim, int32_t v_dim, int32_t block_size,
                   int32_t num_blocks, int32_t chunk, float scale, float softcap, int32_t dtype,
                   void *stream);

/* The same under any nva_mask (workspace: as above with chunk = span), with
 * sinks (fp32 [num_heads], may be NULL): the sum of a head's weights also contains exp(sink), which has no key,
 * bias_slope, bias_rate (fp32 [num_heads], both or neither NULL; not beside a softcap): a key that lies d back has
 * slope * ln(1 + rate * d) taken off its score, and
 * gate ([n_tokens, num_heads], row stride in elements, may be NULL): a head's result times sigmoid(gate). */
int nva_masked_attn(const void *q, int64_t q_row_stride, const void *k_cache, const void *v_cache,
                    const int32_t *block_tables, int64_t bt_row_stride, int32_t max_blocks,
                    const int32_t *cu_seqlens_q, const int32_t *seq_lens, const int32_t *token_seq, void *out,
                    void *workspace, size_t workspace_bytes,
                    int32_t n_tokens, int32_t n_seqs, int32_t max_seqlen_q, int32_t num_heads,
                    int32_t num_kv_heads, int32_t qk_dim, int32_t v_dim, int32_t block_size,
                    int32_t num_blocks, int32_t mask, int32_t span, float scale, float softcap, const float *sinks,
                    const float *bias_slope, const float *bias_rate, const void *gate, int64_t gate_row_stride, int32_t dtype,
                    void *stream);

/* q, k and v of an attention layer, between projection and attention.  x: [n_tokens, num_heads * qk_dim | num_kv_heads *
 * qk_dim | num_kv_heads * v_dim] (row stride in elements) plus bias (as many elements, may be NULL); then RMS norms of q and
 * k, of every head by itself (weights [qk_dim]) or over all heads at once (weights [num_heads * qk_dim] and
 * [num_kv_heads * qk_dim]; a NULL weight: no norm, unless norms, of enum nva_qkv_norms, asks for one without a weight), and of
 * every head's values where norms asks for it; then rotation of the first rot_dims elements of every head by the
 * row's position (pairs i, i + rot_dims / 2; rope_cache as above).  q to q_out [n_tokens, num_heads * qk_dim], k and v to their
 * cache slots.  Caches NULL: the queries only (x then has num_heads * qk_dim columns). */
int nva_qkv_prepare(const void *x, int64_t x_row_stride, const void *bias, const void *q_norm_weight, const void *k_norm_weight,
                    int32_t norms, const float *rope_cache, void *q_out, void *k_cache, void *v_cache,
                    const int32_t *slot_mapping, int64_t num_slots, const int32_t *cu_seqlens_q, const int32_t *seq_lens,
                    const int32_t *token_seq, int32_t n_tokens, int32_t n_seqs, int32_t num_heads, int32_t num_kv_heads,
                    int32_t qk_dim, int32_t v_dim, int32_t rot_dims, int32_t max_position, float eps, int32_t dtype, void *stream);

/* Retention: S_t = decay S_{t-1} + k_t v_t^T, o_t = S_t^T q_t per head, with rotary q and k, k scaled by
 * k_scale; out = o / rms(o) * silu(gate).
 * qkvg: [n_tokens, 2 * num_heads * (qk_dim + v_dim)] (q | k | v | gate, row stride in elements);
 * state: fp32 [num_state_slots, num_heads, qk_dim, v_dim], carried across calls; log2_decay: fp32
 * [num_heads], log2 of every head's decay; rope_cache as above; out: [n_tokens, num_heads * v_dim] dense.
 * workspace: states between the segments of long portions, nva_retention_workspace_bytes() bytes, 16-byte
 * aligned (NULL where that is 0, and for single tokens); needs no initialisation.  max_seqlen_q: longest
 * portion. */
size_t nva_retention_workspace_bytes(int32_t n_seqs, int32_t max_seqlen_q, int32_t num_heads, int32_t qk_dim,
                                     int32_t v_dim, int32_t rot_dims, int32_t dtype);
int nva_retention(const void *qkvg, int64_t row_stride, float *state, const int32_t *state_slots_of_seq,
                  const int32_t *cu_seqlens_q, const int32_t *seq_lens,
                  const float *rope_cache, const float *log2_decay, void *out, void *workspace,
                  size_t workspace_bytes, int32_t n_tokens, int32_t n_seqs,
                  int32_t max_seqlen_q, int32_t num_heads, int32_t qk_dim, int32_t v_dim, int32_t rot_dims,
                  int32_t max_position, int32_t num_state_slots, float k_scale, float eps, int32_t dtype,
                  void *stream);

/*
 * ---- layered models whose mixer and feed-forward branch off one point of the stream ---------
 * Same conventions for rows, dtypes, slots and padded rows as the mixers above.
 */

/* residual[r] = table[ids[r]] * scale (fp32); out1[r] = residual[r] / rms * (weight_offset + weight1), out2 the
 * same with weight2 (weight2 may be NULL: one norm; both NULL: out1 is the residual itself, rounded).  rms = sqrt(mean(x^2) + eps).  out1 has a row stride in elements; copy (may be
 * NULL, row stride likewise): the residual itself, rounded, as well.  clear (may be NULL):
 * clear_count int32 counters set to zero, for a router that runs behind this. */
int nva_embed_rms_norms(const int64_t *ids, const void *table, float scale, const void *weight1, const void *weight2,
                        float weight_offset, float *residual, void *out1, int64_t out1_row_stride, void *out2, void *copy,
                        int64_t copy_row_stride, int32_t *clear, int32_t clear_count, int32_t rows, int32_t width, int32_t vocab,
                        float eps, int32_t dtype, void *stream);

/* residual[r] += mult * (gain1 * y1[r] + gain2 * sum_k term_weight[r, k] * y2[r * terms + k]), in place, fp32; then
 * the norms as above.  y1 or y2, either gain ([width]) and term_weight (fp32) may be NULL (absent; one; one).
 * rows_of (int32 [rows], may be NULL): out[r] is computed from row rows_of[r] (clamped to [0, src_rows)) and
 * residual is not written; without it rows == src_rows. */
int nva_branches_rms_norms(const void *y1, int64_t y1_row_stride, const void *gain1, const void *y2,
                           const float *term_weight, int32_t terms, const void *gain2, float mult, float *residual,
                           const void *weight1, const void *weight2, float weight_offset, void *out1, void *out2,
                           const int32_t *rows_of, int32_t *clear, int32_t clear_count, int32_t rows,
                           int32_t src_rows, int32_t width, float eps, int32_t dtype, void *stream);

/* Layers that norm what a sublayer gives: y[r] = y1_weight[r] * y1[r] + sum_k term_weight[r, k] * y2[r * terms + k];
 * residual[r] += y[r] / rms * (weight_offset + post_weight), in place, fp32; out[r] = residual[r], rounded, or with
 * next_weight residual[r] / rms * (weight_offset + next_weight).  y1_weight (one per row) and term_weight are fp32 with
 * weight_row_stride elements between rows; either may be NULL (one).  The rest as above. */
int nva_post_rms_norms(const void *y1, int64_t y1_row_stride, const float *y1_weight, const void *y2,
                       const float *term_weight, int64_t weight_row_stride, int32_t terms, const void *post_weight,
                       float *residual, const void *next_weight, float weight_offset, void *out, const int32_t *rows_of,
                       int32_t *clear, int32_t clear_count, int32_t rows, int32_t src_rows, int32_t width, float eps,
                       int32_t dtype, void *stream);

/* Branches behind gates of every element: residual[r] += sigmoid(gate[r, :width] + gate_bias[:width]) * y1[r] + sigmoid(gate[r, width:] +
 * gate_bias[width:]) * sum_k y2[r * terms + k], in place, fp32 (y2 may be NULL; gate and gate_bias then need their first width
 * elements only); out[r] = residual[r] / rms * (weight_offset + weight), or, weight NULL, the residual itself, rounded.  gate
 * and out have row strides in elements.  The rest as above. */
int nva_gated_rms_norm(const void *y1, int64_t y1_row_stride, const void *y2, int32_t terms, const void *gate,
                       int64_t gate_row_stride, const void *gate_bias, float *residual, const void *weight, float weight_offset,
                       void *out, int64_t out_row_stride, const int32_t *rows_of, int32_t *clear, int32_t clear_count,
                       int32_t rows, int32_t src_rows, int32_t width, float eps, int32_t dtype, void *stream);

/* A stream that begins anew: residual[r] = product[r] (fp32, dense) + step; out[r] = residual[r] / rms * (weight_offset + weight). */
int nva_entry_rms_norm(const float *product, const void *step, float *residual, const void *weight, float weight_offset, void *out,
                       int32_t *clear, int32_t clear_count, int32_t rows, int32_t width, float eps, int32_t dtype, void *stream);

/* out[r, g] = W_g x[r, g] for every row and group: x + r * x_row_stride + g * x_group_stride, weight [groups, n_out, k_in],
 * out + r * out_row_stride + g * out_group_stride (elements).  out_dtype fp32 keeps the fp32 sums of bf16 products.
 * squared_relu: out = max(., 0)^2. */
int nva_grouped_linear(const void *x, int64_t x_row_stride, int64_t x_group_stride, const void *weight, void *out,
                       int64_t out_row_stride, int64_t out_group_stride, int32_t rows, int32_t groups, int32_t n_out,
                       int32_t k_in, int32_t squared_relu, int32_t dtype, int32_t out_dtype, void *stream);

/* Router of a mixture of experts: logits = weight x + bias (fp32; bias may be NULL), softmax over all experts, the `top` best (ties: the lower
 * index) in descending order, their scores divided by their sum (+ 1e-20) and multiplied by scale.
 * (With scale 1 the weights are the softmax over the chosen logits.)  score (enum nva_score) sigmoid: the chosen logits' sigmoids times
 * scale instead.  weight: [experts + gates, width]; the gates are outputs
 * beside the experts' whose sigmoids follow the choices' weights in every row.
 * choice int32 [rows, top], choice_weight fp32 [rows, top + gates].  lists int32 [experts, list_stride], counts int32 [experts]: the
 * assignments row * top + k of every expert, in no particular order; counts must be zero on entry;
 * list_stride >= rows.  experts <= 1024, gates <= 64, top <= 128. */
int nva_router(const void *x, int64_t x_row_stride, const void *weight, const float *bias, int32_t *choice,
               float *choice_weight, int32_t *lists, int32_t *counts, int64_t list_stride, int32_t rows, int32_t width,
               int32_t experts, int32_t gates, int32_t top, int32_t score, float scale, int32_t dtype, void *stream);

/* out[p] = W_e x[p / terms] (x_per_row) or W_e x[p], for every assignment p of lists to its expert e.
 * weight: [experts, n_out, k_in], or gated: [experts, 2 n_out, k_in] (gate | up) and, with g = min(gate, gate_limit)
 * and u = clamp(up, gate_limit), out = g * sigmoid(gate_slope * g) * (u + gate_shift) (infinity, 1, 0: silu(gate) * up).
 * in_weight (gated only; fp32 [rows, terms], row stride in elements, may be NULL): of what an assignment's expert reads; the products
 * are multiplied by it ahead of the form.  out: [rows * terms, n_out] dense. */
int nva_routed_linear(const void *x, int64_t x_row_stride, const void *weight, void *out, const int32_t *lists,
                      const int32_t *counts, int64_t list_stride, int32_t rows, int32_t terms, int32_t experts,
                      int32_t n_out, int32_t k_in, int32_t x_per_row, int32_t gated, float gate_limit, float gate_slope,
                      float gate_shift, const float *in_weight, int64_t in_weight_row_stride, int32_t dtype, void *stream);

/* The same for few rows, bf16, and in the same launch the product of an expert that every row runs: shared_out[r] = W
 * shared_x[r], shared_weight [shared_n_out, shared_k_in], or gated [2 shared_n_out, shared_k_in] in the same form with
 * a limit of its own; shared_out [rows, shared_n_out] dense.  Inner sizes and row strides are multiples of 8. */
int nva_routed_shared_linear(const void *x, int64_t x_row_stride, const void *weight, void *out, const int32_t *lists,
                             const int32_t *counts, int64_t list_stride, int32_t rows, int32_t terms, int32_t experts,
                             int32_t n_out, int32_t k_in, int32_t x_per_row, int32_t gated, float gate_limit, float gate_slope,
                             float gate_shift, const void *shared_x, int64_t shared_x_row_stride, const void *shared_weight,
                             void *shared_out, int32_t shared_n_out, int32_t shared_k_in, float shared_gate_limit, void *stream);

/* Latent attention, what a row leaves behind and its query latent.
 * x: [n_tokens, q_rank | kv_rank | rot_dim] (row stride in elements).
 * q_out [n_tokens, q_rank] = first part / rms * q_norm_weight; cache row slot_mapping[i] of [num_slots, kv_rank + rot_dim] =
 * (second part / rms * kv_norm_weight | third part, neighbours (2i, 2i + 1) rotated by the row's position).
 * q_rank 0: no query latent (q_out and its weight are not used).  cache NULL: the queries only (x then has q_rank columns).  rope_cache: fp32 [max_position, rot_dim], cos in the
 * first half of a row, sin in the second. */
int nva_latent_prepare(const void *x, int64_t x_row_stride, const void *q_norm_weight, const void *kv_norm_weight,
                       const float *rope_cache, void *q_out, void *cache, const int32_t *slot_mapping, int64_t num_slots,
                       const int32_t *cu_seqlens_q, const int32_t *seq_lens, const int32_t *token_seq, int32_t n_tokens,
                       int32_t n_seqs, int32_t q_rank, int32_t kv_rank, int32_t rot_dim, int32_t max_position, float eps,
                       int32_t dtype, void *stream);

/* Absorbed form: the query at position p meets the cached rows (p - window, p] of its sequence,
 *   score = (q_latent . c + rotate(q_rot) . k_rot) * scale,  out = sigmoid(gate) * sum softmax(score) c.
 * gate may be NULL (one); sinks (fp32 [num_heads], may be NULL): the sum of a head's weights also contains exp(sink).
 * q_latent [n_tokens, num_heads, kv_rank] dense; q_rot [n_tokens, num_heads, rot_dim], not yet rotated; gate
 * [n_tokens, num_heads] logits; cache [num_blocks, block_size, kv_rank + rot_dim]; out [n_tokens, num_heads, kv_rank] dense.
 * A key behind a table entry outside [0, num_blocks) is not seen.  kv_rank + rot_dim <= 1024.
 * workspace: partial results, nva_latent_attn_workspace_bytes() bytes, 16-byte aligned (NULL where that is 0). */
size_t nva_latent_attn_workspace_bytes(int32_t n_tokens, int32_t num_heads, int32_t kv_rank, int32_t rot_dim,
                                       int32_t max_blocks, int32_t block_size, int32_t window, int32_t dtype);
int nva_latent_attn(const void *q_latent, const void *q_rot, int64_t qr_row_stride, int64_t qr_head_stride, const void *gate,
                    int64_t gate_row_stride, const float *sinks, const float *rope_cache, const void *cache, const int32_t *block_tables,
                    int64_t bt_row_stride, int32_t max_blocks, const int32_t *cu_seqlens_q, const int32_t *seq_lens,
                    const int32_t *token_seq, void *out, void *workspace, size_t workspace_bytes, int32_t n_tokens,
                    int32_t n_seqs, int32_t num_heads, int32_t kv_rank, int32_t rot_dim, int32_t block_size,
                    int32_t num_blocks, int32_t window, int32_t max_position, float scale, int32_t dtype, void *stream);

/* Expanded form, for portions.  nva_latent_gather copies the cache rows of the last key_cu[s + 1] - key_cu[s] tokens of
 * every sequence s to out [n_keys, row_width]; the caller multiplies the latents out to kv [n_keys, num_heads * dim |
 * num_heads * v_dim]; nva_latent_prefill attends:
 *   score = (q[:dim] . k + rotate(q[dim:]) . k_rot) * scale,  out = sigmoid(gate) * sum softmax(score) v
 * over the positions (p - window, p] that were gathered, gate and sinks as above.  q [n_tokens, num_heads, dim + rot_dim], bf16 only, sizes
 * multiples of 8 (nva_latent_prefill_supported). */
int nva_latent_gather(const void *cache, const int32_t *block_tables, int64_t bt_row_stride, int32_t max_blocks,
                      const int32_t *key_cu, const int32_t *seq_lens, void *out, int32_t n_keys, int32_t n_seqs,
                      int32_t row_width, int32_t block_size, int32_t num_blocks, int32_t dtype, void *stream);
int nva_latent_prefill_supported(int32_t dim, int32_t rot_dim, int32_t v_dim, int32_t dtype);
int nva_latent_prefill(const void *q, int64_t q_row_stride, const void *kv, int64_t kv_row_stride, const void *k_rot,
                       int64_t kr_row_stride, const void *gate, int64_t gate_row_stride, const float *sinks, const float *rope_cache,
                       const int32_t *cu_seqlens_q, const int32_t *seq_lens, const int32_t *key_cu, void *out,
                       int32_t n_tokens, int32_t n_seqs, int32_t max_seqlen_q, int32_t num_heads, int32_t dim, int32_t rot_dim,
                       int32_t v_dim, int32_t window, int32_t max_position, float scale, int32_t dtype, void *stream);

/* Matrix memory with exponential gates, head norm and output gate.  With i = cap tanh((z_i + b_i) / cap) and
 * f = log sigmoid(cap tanh((z_f + b_f) / cap)):  m_t = max(f + m_{t-1}, i),  S_t = e^{f + m_{t-1} - m_t} S_{t-1} +
 * e^{i - m_t} k v^T,  n_t likewise with k,  o = S_t^T q / (max(|n_t . q|, e^{-m_t}) + 1e-6), q scaled by q_scale;
 * out = o / rms(o) * norm_weight * sigmoid(gate).
 * qkvg: [n_tokens, 2 * num_heads * (qk_dim + v_dim)] (q | k | v | gate, row stride in elements); gate_logits fp32
 * [n_tokens, 2 * num_heads] dense (input gates | forget gates), gate_bias fp32 [2 * num_heads], norm_weight
 * [num_heads * v_dim]; state / mass / top: fp32 [num_state_slots, num_heads, (qk_dim, v_dim | qk_dim | -)], carried across
 * calls; out: [n_tokens, num_heads * v_dim] dense.  workspace: states between the segments of long portions,
 * nva_mlstm_workspace_bytes() bytes, 16-byte aligned (NULL where that is 0, and for single tokens). */
size_t nva_mlstm_workspace_bytes(int32_t n_seqs, int32_t max_seqlen_q, int32_t num_heads, int32_t qk_dim, int32_t v_dim,
                                 int32_t dtype);
int nva_mlstm(const void *qkvg, int64_t row_stride, const float *gate_logits, const float *gate_bias,
              const void *norm_weight, float *state, float *mass, float *top, const int32_t *state_slots_of_seq,
              const int32_t *cu_seqlens_q, const int32_t *seq_lens, void *out, void *workspace,
              size_t workspace_bytes, int32_t n_tokens, int32_t n_seqs, int32_t max_seqlen_q, int32_t num_heads,
              int32_t qk_dim, int32_t v_dim, int32_t num_state_slots, float q_scale, float gate_cap, float eps,
              int32_t dtype, void *stream);

/*
 * Calibration, no counterpart in the reference: streams nbytes from src with the access discipline of
 * the decode kernel (2048 wavefront workers, contiguous slices, 16-byte non-temporal loads) and keeps
 * nothing.  Its duration is what any kernel that reads that many bytes needs at least on this GPU;
 * bench.py reports it next to the roofline fractions.  src 16-byte aligned, nbytes % 16 == 0; sink:
 * at least 4 writable bytes of device memory (practically never written).
 */
int nva_probe_stream_read(const void *src, int64_t nbytes, void *sink, void *stream);

#ifdef __cplusplus
}
#endif
#endif /* NANOVLLM_AMD_H */
