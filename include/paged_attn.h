/*
 * paged_attn.h - C ABI of libpaged_attn.so: paged-KV attention for one MI355X
 * (gfx950) behind the attention / KV-cache call surface of the `rollouts`
 * inference engine.
 *
 * Conventions for every entry point
 *   - plain pointers and sizes; device pointers unless the name says host;
 *   - `stream` is a hipStream_t passed as void* (NULL = the null stream);
 *     work is enqueued asynchronously on it, nothing synchronises;
 *   - the return value is a status: PA_OK, or a negative PA_ERR_* after which
 *     pa_last_error() (thread-local text) says what was wrong.  Arguments are
 *     checked on the host before any HIP call, so a rejected call has touched
 *     neither the GPU nor its buffers;
 *   - the library allocates nothing: the caller owns inputs, outputs and the
 *     decode workspace;
 *   - indices read from device memory (slots, block ids) are range-checked by
 *     the kernels against `total_slots` / `num_blocks`: an out-of-range index
 *     is skipped (append) or reads as zeros (gather, attention), never a fault.
 *
 * Pool layout (fixed by the reference, attention/config.py:43-45, one layer's
 * slice): element [slot][kv_head][d] at ((slot*num_kv_heads)+kv_head)*head_dim+d,
 * slot = block_id*block_size + offset_in_block.
 *
 * Reference citations are relative to rollouts/rollouts/inference/.
 */
#ifndef PAGED_ATTN_H
#define PAGED_ATTN_H

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

#define PA_OK 0
#define PA_ERR_INVALID_ARG (-1) /* NULL pointer, negative size, inconsistent dims */
#define PA_ERR_UNSUPPORTED (-2) /* dtype / head_dim / group size has no kernel */
#define PA_ERR_WORKSPACE (-3)   /* decode workspace missing or too small */
#define PA_ERR_HIP (-4)         /* a HIP launch reported an error */

/* element types of q / out / the KV pool */
#define PA_F32 0
#define PA_BF16 1
#define PA_F16 2
#define PA_FP8_E4M3 3 /* OCP e4m3fn, KV pool only; q/out stay 16- or 32-bit */

/* Library ABI version (bumped when an entry point is added or a signature or contract changes; now 9). */
int pa_version(void);

/* Text of the calling thread's most recent error; "" if none. */
const char *pa_last_error(void);

/* Bytes per element of a PA_* dtype, or 0 for an unknown code. */
int pa_dtype_bytes(int dtype);

/*
 * KV append / scatter.  Replaces FlexAttentionBackend._store_kv
 * (attention/flex_backend.py:116-142):
 *     for i in range(n_tokens): s = slots[i]
 *         if s >= 0: k_cache[s] = k_src[i]; v_cache[s] = v_src[i]
 * A pure byte copy of rows of num_kv_heads*head_dim elements; rows whose slot
 * is negative (the reference's filter, :139-142) or >= total_slots are
 * dropped.  Duplicate slots in one call: which source row wins is unspecified
 * (as for the reference's index_put on a GPU).
 *   k_cache,v_cache : one layer's pool slice, [total_slots][row]
 *   k_src,v_src     : [n_tokens][row], contiguous
 *   slots           : int64[n_tokens]
 *   elem_bytes      : 1, 2 or 4; row bytes must be a multiple of 4
 */
int pa_kv_scatter(void *k_cache, void *v_cache, const void *k_src, const void *v_src,
                  const int64_t *slots, int64_t n_tokens, int64_t total_slots,
                  int num_kv_heads, int head_dim, int elem_bytes, void *stream);

/*
 * Block-table gather.  Replaces FlexAttentionBackend._gather_kv_from_cache
 * (attention/flex_backend.py:233-279):
 *     out[b][pos] = cache[bt[b][pos / bs] * bs + pos % bs]   for pos < seq_lens[b]
 * and zeros for pos >= seq_lens[b], for positions whose block-table entry is
 * missing (the reference's short-table case, :274; here: entry < 0, entry >=
 * num_blocks, or pos / bs >= bt_stride), up to max_len.  Bit-exact copy.
 *   block_tables : int32[batch][bt_stride], row-padded with -1
 *   seq_lens     : int32[batch]
 *   k_out,v_out  : [batch][max_len][row], every byte is written
 */
int pa_kv_gather(const void *k_cache, const void *v_cache, void *k_out, void *v_out,
                 const int32_t *block_tables, int64_t bt_stride, const int32_t *seq_lens,
                 int batch, int64_t max_len, int64_t num_blocks, int block_size,
                 int num_kv_heads, int head_dim, int elem_bytes, void *stream);

/*
 * Workspace of pa_decode in bytes (host arithmetic only, no GPU call); 0 on
 * error.  pa_decode splits the batch's pool blocks evenly over a machine-sized
 * grid of workgroups; a sequence whose blocks fall into several workgroups
 * leaves one partial result per piece in the workspace.  The size depends on
 * the shapes only, never on the sequence lengths, so one allocation serves
 * every step of a model.  Alignment: 256 bytes.  The first
 * PA_DECODE_TICKET_BYTES bytes hold the arrival counters of the merge inside
 * the split pass: zero-fill them once after allocating the workspace (before
 * its first use; outside any stream capture) and leave them to the library
 * afterwards - every call returns them to "nothing arrived", whatever its
 * shapes, so captured graphs replay without clearing anything.  The rest need
 * not be initialised.  Calls that share a workspace must not overlap in time.
 */
#define PA_DECODE_TICKET_BYTES (640u << 10)
size_t pa_decode_workspace_bytes(int batch, int num_q_heads, int num_kv_heads, int head_dim,
                                 int kv_dtype);

/*
 * Kernel launches one pa_decode call of these shapes makes on the current device: 1 when the batch is large
 * enough that the split pass merges a sequence's pieces itself, else 2 (split pass, reduction pass); negative on
 * error.  For callers that time or profile the passes.  (No counterpart in the reference.)
 */
int pa_decode_passes(int batch, int num_q_heads, int num_kv_heads, int head_dim, int kv_dtype);

/*
 * Paged decode attention.  Replaces FlexAttentionBackend._decode_attention
 * (attention/flex_backend.py:187-231) together with the gather and the GQA
 * repeat_interleave it performs: for sequence b and query head h
 *     kvh = h / (num_q_heads / num_kv_heads)
 *     out[b][h] = softmax_j( scale * q[b][h] . K[b][j][kvh] ) . V[b][j][kvh],  j < seq_lens[b]
 * with K/V rows addressed through the block table as in pa_kv_gather; a
 * position whose block-table entry is missing acts as an all-zero key and
 * value (logit 0), as it does in the reference.  Accumulation is fp32.  All
 * integer inputs stay on the device: the host never reads seq_lens.
 *   q, out        : [batch][num_q_heads][head_dim], dtype q_dtype, 16-byte aligned
 *   head_dim      : a multiple of 8 up to 256 (of 16 for an fp8 pool; rows of whole 16-byte vectors); the
 *                   reference takes any head_dim (attention/config.py:22-24)
 *   kv_dtype      : q_dtype, or PA_FP8_E4M3 with k_scale/v_scale =
 *                   float[num_blocks][num_kv_heads] (value = fp8 * scale)
 *   extra_zero_keys: NULL, or int32[batch]: that many additional all-zero
 *                   keys take part in sequence b's softmax.  The reference
 *                   zero-pads ragged batches to the longest sequence without a
 *                   mask (:253-264, :227-229); passing max_len - seq_lens[b]
 *                   reproduces it.
 *   window        : 0; negative: chunks of -window positions counted from the sequence's start, of which a query sees
 *                   its own (keys j <= p of the same chunk; no counterpart in the reference); or positive, a
 *                   sliding window: only the last `window` keys of each sequence are attended
 *                   (j >= seq_lens[b] - window), the rule of the reference's causal_sliding_window_mask
 *                   (attention/mask.py:83-89: q_idx - kv_idx < window_size) for the query at position
 *                   seq_lens[b]-1; blocks wholly before the window are never read.  The reference's own
 *                   decode applies a window only through a caller-built ctx.block_mask
 *                   (flex_backend.py:220-225).  Not combinable with extra_zero_keys.
 *   batch         : any; more than 8192 sequences are taken 8192 at a time, one after the other on the stream
 *   workspace     : pa_decode_workspace_bytes(...) bytes, its first PA_DECODE_TICKET_BYTES zero-filled once
 *   A sequence of length 0 yields zeros.
 */
int pa_decode(const void *q, const void *k_cache, const void *v_cache, void *out,
              const int32_t *block_tables, int64_t bt_stride, const int32_t *seq_lens,
              const int32_t *extra_zero_keys, const float *k_scale, const float *v_scale,
              int batch, int num_q_heads, int num_kv_heads, int head_dim, int block_size,
              int64_t num_blocks, float scale, int window, int q_dtype, int kv_dtype, void *workspace,
              size_t workspace_bytes, void *stream);

/*
 * The two passes of pa_decode as separate calls, same arguments:
 * pa_decode_split followed by pa_decode_reduce on the same stream and
 * workspace give pa_decode's result (to rounding: for large batches pa_decode
 * merges inside its one launch, in another order; see pa_decode_passes).  For
 * callers that time or schedule the passes separately.  (The
 * reference has one fused call site, attention/flex_backend.py:227-229; these
 * have no separate counterpart there.)
 */
int pa_decode_split(const void *q, const void *k_cache, const void *v_cache, void *out,
                    const int32_t *block_tables, int64_t bt_stride, const int32_t *seq_lens,
                    const int32_t *extra_zero_keys, const float *k_scale, const float *v_scale,
                    int batch, int num_q_heads, int num_kv_heads, int head_dim, int block_size,
                    int64_t num_blocks, float scale, int window, int q_dtype, int kv_dtype, void *workspace,
                    size_t workspace_bytes, void *stream);
int pa_decode_reduce(const void *q, const void *k_cache, const void *v_cache, void *out,
                     const int32_t *block_tables, int64_t bt_stride, const int32_t *seq_lens,
                     const int32_t *extra_zero_keys, const float *k_scale, const float *v_scale,
                     int batch, int num_q_heads, int num_kv_heads, int head_dim, int block_size,
                     int64_t num_blocks, float scale, int window, int q_dtype, int kv_dtype, void *workspace,
                     size_t workspace_bytes, void *stream);

/*
 * pa_decode without a workspace argument and without any allocation, for callers that cannot allocate device
 * memory: code under HIP graph capture, serving loops with a fixed memory plan, harnesses that forbid
 * hipMalloc.  (No counterpart in the reference, which allocates freely inside its decode,
 * attention/flex_backend.py:253-264.)  The partial results of the split pass go to a scratch array of
 * PA_DECODE_STATIC_SCRATCH_BYTES that the library's code object holds on every GPU it is loaded on, from load
 * until the process ends.  Arguments and results are those of pa_decode, bit for bit.
 *   - Shapes whose partials do not fit return PA_ERR_WORKSPACE (the message gives the bytes needed); the
 *     need is (workgroups of the split pass + planes * batch) * heads * (head_dim + 2) * 4 bytes, e.g.
 *     8.5 MB for batch 256, 32 query / 8 kv heads of 128 on a 256-CU device.
 *   - Every call on one GPU shares that GPU's array, which keeps the previous call's partials: calls whose
 *     kernels may overlap on one GPU (different streams, different threads) race; order them.
 *   - The first call on a device asks the runtime for the array's address (hipGetSymbolAddress); make that
 *     call outside a stream capture.  No call allocates or frees.
 */
#define PA_DECODE_STATIC_SCRATCH_BYTES (16u << 20)
int pa_decode_static(const void *q, const void *k_cache, const void *v_cache, void *out,
                     const int32_t *block_tables, int64_t bt_stride, const int32_t *seq_lens,
                     const int32_t *extra_zero_keys, const float *k_scale, const float *v_scale, int batch,
                     int num_q_heads, int num_kv_heads, int head_dim, int block_size, int64_t num_blocks,
                     float scale, int window, int q_dtype, int kv_dtype, void *stream);

/*
 * Causal prefill attention over a paged context.  Covers both
 * FlexAttentionBackend._prefill_attention (attention/flex_backend.py:144-185,
 * the is_causal SDPA over the step's own K/V) and chunked prefill over cached
 * prefix blocks (a composition the reference does not have): for sequence b
 * the q_lens[b] query rows are the LAST q_lens[b] positions of a context of
 * ctx_lens[b] keys, and row i attends keys j <= ctx_lens[b] - q_lens[b] + i.
 * The keys are read through the block table, so the step's new K/V must have
 * been appended (pa_kv_scatter) first.  Sequences that list the same block
 * ids share those blocks.
 *   q, out   : [total_q][num_q_heads][head_dim] packed rows, sequence b's rows
 *              start at q_starts[b]; dtype PA_BF16 or PA_F16 (MFMA path) or
 *              PA_F32 (vector path)
 *   head_dim : a multiple of 8 up to 256.  bf16 / fp16 run on the matrix cores: 32, 64, 128 and 256 have
 *              kernels of their own, every other multiple of 8 runs the kernel of the next larger size (rows in
 *              memory keep their length); PA_F32 runs on the vector kernel
 *   ctx_lens, q_lens, q_starts : int32[batch]
 *   max_q_len: upper bound of q_lens (grid sizing)
 *   window   : 0; negative: chunks of -window positions, as in pa_decode; or the sliding window of CacheConfig.sliding_window (attention/config.py:31): row i at
 *              position p = ctx_lens[b] - q_lens[b] + i attends keys p - window < j <= p
 *              (attention/mask.py:83-89); tiles wholly before the window of a workgroup's rows are not loaded.
 *   row_first_key : NULL, or int32[total_q] indexed like the rows of q: the first key position (in the
 *              row's own sequence) the row attends, on top of the causal bound -- the packed-document mask
 *              of create_document_mask (attention/mask.py:141-191: same document and q_idx >= kv_idx) with
 *              row_first_key = start of the row's document.  Must not decrease along a sequence; values
 *              are clamped to [0, position of the row], so a row always sees itself.  Combines with window
 *              (the later of the two bounds applies).
 */
int pa_prefill_paged(const void *q, const void *k_cache, const void *v_cache, void *out,
                     const int32_t *block_tables, int64_t bt_stride, const int32_t *ctx_lens,
                     const int32_t *q_lens, const int32_t *q_starts, const int32_t *row_first_key,
                     int batch, int max_q_len, int num_q_heads, int num_kv_heads, int head_dim,
                     int block_size, int64_t num_blocks, float scale, int window, int dtype, void *stream);

/*
 * pa_prefill_paged with a workspace, for launches of few query rows.  The reference's SDPA call
 * (attention/flex_backend.py:180-182) spreads one long row's keys over the machine however PyTorch likes; the
 * matrix-core kernels here give a workgroup 256 row-head pairs and all their keys, so one 2048-row chunk behind a
 * long cached context occupies a quarter of the compute units.  Given a workspace, such a launch cuts every
 * workgroup's keys into up to 8 pieces run by workgroups of their own, which leave (maximum, sum, unnormalised
 * output row) per piece in the workspace, and a second kernel merges them - the arithmetic of pa_decode's
 * reduction pass.  Results equal pa_prefill_paged's to fp32 merge-order rounding.
 *   total_q        : rows of q / out (every q_starts[b] + q_lens[b] <= total_q)
 *   workspace      : pa_prefill_workspace_bytes(...) bytes, 256-byte aligned, contents need not be initialised;
 *                    NULL or too small for any split: the call is pa_prefill_paged.  A smaller workspace is used
 *                    for as many pieces as it holds.
 * pa_prefill_workspace_bytes: what the split the library would choose for these shapes on the current device needs
 * (0 when the launch fills the device anyway, or for fp32, which only the unsplit vector kernel takes; a head size
 * between 32 / 64 / 128 / 256 is sized for partial rows of the next larger one); host arithmetic plus one
 * device-attribute query.
 * bt_stride * block_size bounds the context length the split is sized for.
 */
size_t pa_prefill_workspace_bytes(int batch, int max_q_len, int64_t total_q, int64_t bt_stride, int block_size,
                                  int window, int num_q_heads, int num_kv_heads, int head_dim, int dtype);
int pa_prefill_paged_ws(const void *q, const void *k_cache, const void *v_cache, void *out,
                        const int32_t *block_tables, int64_t bt_stride, const int32_t *ctx_lens,
                        const int32_t *q_lens, const int32_t *q_starts, const int32_t *row_first_key,
                        int batch, int max_q_len, int num_q_heads, int num_kv_heads, int head_dim,
                        int block_size, int64_t num_blocks, float scale, int window, int dtype, void *stream,
                        int64_t total_q, void *workspace, size_t workspace_bytes);

/*
 * Attention under an arbitrary mask: what FlexAttentionBackend does with a ctx.block_mask built from any
 * mask_mod(b, h, q_idx, kv_idx) predicate (attention/flex_backend.py:170-178 in prefill, :220-225 in decode;
 * predicates such as attention/mask.py:42, :84, :171).  The caller evaluates the predicate into bits; row r of
 * sequence b (packed row q_starts[b] + r), query head h attends key j < n_keys iff bit j of its mask row is
 * set - nothing else is implied, a causal bound included.  Keys j >= ctx_lens[b] and keys in absent blocks are
 * zero rows (logit 0, zero value), which is what the reference's zero-padded decode gather hands to
 * flex_attention (:253-264); a row with no bit set gives zeros.
 *   q, out  : [total_q][num_q_heads][head_dim], dtype F32 / BF16 / F16
 *   kv_dtype: dtype, or PA_FP8_E4M3 (16-bit q) with k_scale / v_scale float[num_blocks][num_kv_heads] as in pa_decode
 *   mask    : uint32 [total_q][mask_heads][mask_words], bit j of word j/32; mask_heads is 1 (all heads share
 *             the row) or num_q_heads
 * The general path, not a fast one: one workgroup per (head, row), a wave-wide reduction per visible key.  The
 * structured masks (causal, sliding window, packed documents) go through pa_prefill_paged / pa_decode.
 */
int pa_attend_masked(const void *q, const void *k_cache, const void *v_cache, void *out,
                     const int32_t *block_tables, int64_t bt_stride, const int32_t *ctx_lens,
                     const int32_t *q_lens, const int32_t *q_starts, const uint32_t *mask, int mask_heads,
                     int mask_words, int n_keys, int batch, int max_q_len, int num_q_heads, int num_kv_heads,
                     int head_dim, int block_size, int64_t num_blocks, float scale, int dtype, int kv_dtype,
                     const float *k_scale, const float *v_scale, void *stream);

/*
 * pa_prefill_paged evaluated by the vector kernel (one workgroup per query row, the decode inner loop) whatever
 * the element type: the path fp32 and fp8-pool calls take anyway, selectable for the 16-bit shapes too so that
 * the two kernels can be checked against each other.  Same arguments, same results to rounding.
 * (No separate counterpart in the reference: both are attention/flex_backend.py:144-185.)
 */
int pa_prefill_paged_rowwise(const void *q, const void *k_cache, const void *v_cache, void *out,
                             const int32_t *block_tables, int64_t bt_stride, const int32_t *ctx_lens,
                             const int32_t *q_lens, const int32_t *q_starts, const int32_t *row_first_key,
                             int batch, int max_q_len, int num_q_heads, int num_kv_heads, int head_dim,
                             int block_size, int64_t num_blocks, float scale, int window, int dtype, void *stream);

/*
 * fp8-e4m3 pool construction (no counterpart in the reference; its oracle is
 * "dequantise, then attend in fp32").  For every (block, kv head):
 *     s = max|x| / 448  (s = 1 when the block is all zero)
 *     dst = e4m3fn_rne(x / s),  scale[block][kv_head] = s
 *   src   : [num_blocks*block_size][num_kv_heads][head_dim], src_dtype F32/BF16/F16
 *   dst   : same shape, one byte per element
 *   scale : float[num_blocks][num_kv_heads]
 */
int pa_quantize_kv_e4m3(const void *src, void *dst, float *scale, int64_t num_blocks,
                        int block_size, int num_kv_heads, int head_dim, int src_dtype,
                        void *stream);

/*
 * Append rows to an fp8-e4m3 pool (no counterpart in the reference: its _store_kv, flex_backend.py:116-142,
 * copies rows of the pool's own type).  Policy, per (block, kv head) tile: "re-round on growth".
 *   - rows of the tile below the lowest offset this call writes are its content so far; a call that writes
 *     offset 0 starts the tile over (recycled blocks need no clearing);
 *   - a_old = scale * max|stored value| over the content, a_new = max|x| over the rows written by this call;
 *   - a_new <= a_old: scale unchanged; otherwise scale' = a_new/448 (1 if a_new = 0) and every content byte
 *     becomes e4m3fn_rne(float(byte) * (scale / scale'));
 *   - new rows are stored as e4m3fn_rne(x / scale').
 *   slots          : int64[n_tokens], slot = block*block_size + offset; negative or out-of-pool slots are skipped;
 *                    of two tokens with the same slot the later one is stored
 *   touched_blocks : int32[n_touched], the distinct blocks the slots fall in (extra entries are harmless,
 *                    a block must not appear twice)
 *   row_order, block_start : optional index of the rows by touched block (both NULL: every workgroup scans the
 *                    whole slot list, n_touched * n_tokens slot reads per tensor, fine for a decode step and
 *                    quadratic in the length of a prefill chunk).  row_order int32[n_tokens]: token indices
 *                    grouped by touched block; block_start int32[n_touched + 1]: tokens
 *                    row_order[block_start[i]] .. row_order[block_start[i+1] - 1] are those whose slots fall in
 *                    touched_blocks[i].  A token the index leaves out is not stored; entries out of range are
 *                    ignored.
 *   k_src, v_src   : [n_tokens][num_kv_heads][head_dim] in src_dtype (F32/BF16/F16)
 *   k_scale,v_scale: float[num_blocks][num_kv_heads], updated in place
 */
int pa_kv_append_e4m3(void *k_cache, void *v_cache, float *k_scale, float *v_scale, const void *k_src,
                      const void *v_src, const int64_t *slots, int64_t n_tokens,
                      const int32_t *touched_blocks, int n_touched, const int32_t *row_order,
                      const int32_t *block_start, int64_t num_blocks, int block_size, int num_kv_heads,
                      int head_dim, int src_dtype, void *stream);

/*
 * Rotary position embedding fused with the KV append: the step a model runs immediately before this path
 * (rollouts/tools/functional_extractor/llama_functional.py:203 applies apply_rotary_pos_emb, :75-98, right
 * before attention, :210) merged with FlexAttentionBackend._store_kv (attention/flex_backend.py:116-142), so
 * the step's new K rows are read once and written once.  For every token i, with r = positions[i] (or i):
 *     x_embed = (x * cos[r]) + (rotate_half(x) * sin[r]),   rotate_half(x) = cat(-x[D/2:], x[:D/2])
 * for every head of q (written to q_out, which may be q itself) and of k; the rotated k row goes to
 * k_cache[slots[i]] (and to k_out[i] when k_out is given), the v row to v_cache[slots[i]].  Every product and
 * the sum are rounded to `dtype`, as when the statement is evaluated on tensors of that type: results equal
 * that evaluation bit for bit.
 *   q, q_out     : [n_tokens][num_q_heads][head_dim]
 *   k_src, v_src : [n_tokens][num_kv_heads][head_dim];  k_out: same shape or NULL
 *   k_cache, v_cache : [total_slots][num_kv_heads][head_dim] of the same dtype
 *   cos, sin     : [rope_rows][head_dim] of the same dtype (both halves are read, as the statement does)
 *   positions    : int32[n_tokens] rows of cos/sin, clamped to the table; NULL: token i uses row i
 *                  (tables laid out per token, the (batch, seq_len, head_dim) form of llama_functional.py:101-136)
 *   slots        : int64[n_tokens]; negative or out-of-pool slots skip the cache write; NULL: no cache write
 *                  (then k_out is required)
 * head_dim/2 elements must fill whole 16-byte vectors (head_dim % 16 == 0 for 16-bit types).
 */
int pa_rope_kv_append(const void *q, void *q_out, const void *k_src, const void *v_src, void *k_out,
                      void *k_cache, void *v_cache, const void *cos, const void *sin, const int32_t *positions,
                      int64_t rope_rows, const int64_t *slots, int64_t n_tokens, int64_t total_slots,
                      int num_q_heads, int num_kv_heads, int head_dim, int dtype, void *stream);

/*
 * The same for an fp8-e4m3 pool: q is rotated to q_out, the k rows are rotated as pa_rope_kv_append does
 * (rounded to src_dtype) while pa_kv_append_e4m3's append reads them, and the v rows are appended as they are.
 * Arguments as in pa_rope_kv_append and pa_kv_append_e4m3; the result equals pa_rope_kv_append into a dense
 * k_out followed by pa_kv_append_e4m3 of k_out, bit for bit.
 */
int pa_rope_kv_append_e4m3(const void *q, void *q_out, const void *k_src, const void *v_src, void *k_cache,
                           void *v_cache, float *k_scale, float *v_scale, const void *cos, const void *sin,
                           const int32_t *positions, int64_t rope_rows, const int64_t *slots, int64_t n_tokens,
                           const int32_t *touched_blocks, int n_touched, const int32_t *row_order,
                           const int32_t *block_start, int64_t num_blocks, int block_size, int num_q_heads,
                           int num_kv_heads, int head_dim, int src_dtype, void *stream);

/*
 * Dequantise listed blocks of an fp8-e4m3 pool into a compact 16-bit pool (no counterpart in the reference):
 * block j of dst = block block_ids[j] of the pool, every value float(byte) * scale[block][kv_head] rounded to
 * dst_dtype (BF16/F16).  Used to run prefill over an fp8 pool on the matrix cores: dequantise the blocks the
 * step's block tables name (each once, however many sequences share it), renumber the tables to positions in
 * block_ids, and call pa_prefill_paged on dst.  Ids outside [0, num_blocks) give zero blocks.
 *   cache : [num_blocks*block_size][num_kv_heads][head_dim] bytes;  scale: float[num_blocks][num_kv_heads]
 *   dst   : [n_ids*block_size][num_kv_heads][head_dim] of dst_dtype;  head_dim % 16 == 0
 */
int pa_dequantize_blocks_e4m3(const void *cache, const float *scale, const int32_t *block_ids, int n_ids,
                              void *dst, int64_t num_blocks, int block_size, int num_kv_heads, int head_dim,
                              int dst_dtype, void *stream);

/*
 * ------------------------------------------------------------------ decoder blocks around attention
 * The entry points below serve decoder blocks other than the reference's Llama block (none of them has a counterpart
 * there): a 32-bit residual stream, layer norm or RMS norm, gated activations, short convolutions ahead of attention,
 * and linear-attention layers with a carried state.  dtype is PA_F32 or PA_BF16, the type of activations and
 * products; residual, norm weights, statistics, angles and states are float whatever the dtype.  A portion is a run of
 * consecutive new rows of one sequence: rows [q_starts[b], q_starts[b] + q_lens[b]) at positions ctx_lens[b] -
 * q_lens[b] ... ctx_lens[b] - 1.  With q_lens and q_starts NULL every sequence brings one row, row b (a decode
 * step); a sequence with ctx_lens[b] = 0 is padding and is skipped.  A portion at position 0 starts from an empty
 * state whatever its slot held before.
 */
#define PA_NORM_NONE 0
#define PA_NORM_LAYER 1
#define PA_NORM_RMS 2
#define PA_ACT_SILU 0
#define PA_ACT_GELU_TANH 1
#define PA_ACT_NONE 2
#define PA_ACT_RELU2 3 /* max(z, 0)^2 (pa_bias_act) */
#define PA_GATE_SIGMOID_LAST 0 /* norm, then sigmoid(gate) */
#define PA_GATE_SILU_FIRST 1   /* silu(gate), then norm */
#define PA_GATE_SILU_LAST 2    /* norm, then silu(gate) */
#define PA_GATE_NONE 3         /* norm only */
#define PA_GL_SSD 0            /* recurrences of pa_gated_linear */
#define PA_GL_MLSTM 1
#define PA_MOE_SIGMOID 0 /* scores of pa_moe_choose */
#define PA_MOE_SOFTMAX 1
#define PA_MOE_NO_SHARED 0
#define PA_MOE_SHARED_GATED 1 /* weight sigmoid(its logit) */
#define PA_MOE_SHARED 2       /* weight 1 */
#define PA_V_PLAIN 0 /* values as they are */
#define PA_V_FIRST 1 /* values as they are, also written to v_first */
#define PA_V_MIX 2   /* (1 - lambda) value + lambda v_first */
#define PA_QKV_TILE_ROWS 16 /* rows of a sequence's portion per tile of pa_qkv_conv_append and pa_short_conv */

/*
 * Residual sum and norm of one row at a time:
 *     x = table[ids[row]] * table_scale             when ids is given (with ids_add, plus x[row]), else x[row]
 *     x += pos_table[positions[row]]                when positions is given (with ids)
 *     x += y                                        when y is given; with y_weight, y / rms(y) * y_weight
 *     out = norm(x) * norm_weight + norm_bias       PA_NORM_LAYER or PA_NORM_RMS; PA_NORM_NONE: x in dtype
 * where rms(v) = sqrt(mean(v^2) + eps) and the layer norm divides by sqrt(variance + eps) with the variance as the
 * mean squared deviation.  x is written back when ids or y is given.  With row_index the call only reads: output
 * row r comes from residual row row_index[r] (< x_rows).  Ids and indices out of range read as zero rows.
 * With mix_weight (float[rows][mix + 1]) y is a weighted sum of rows, taken in 32-bit: sum over i < mix of
 * mix_weight[row][i] y[row * mix + i], plus mix_weight[row][mix] y_extra[row] when y_extra is given.
 * Without mix_weight y may have a y_bias, and with y2 it is the sum of two branches, each normed (with y_eps) on its own:
 * y = y / rms(y) * y_part + y2 / rms(y2) * y2_part, ahead of y_weight's norm.
 *   x : float[rows][width];  y, y2, y_extra, table, pos_table, out : dtype;  weights and bias : float[width] or NULL;  width <= 16384
 */
int pa_residual_norm(float *x, const void *y, const float *mix_weight, int mix, const void *y_extra,
                     const float *y_bias, const void *y2, const float *y_part, const float *y2_part,
                     const float *y_weight, float y_eps, const int64_t *ids, int ids_add, const void *table,
                     int64_t table_rows, float table_scale, const int64_t *positions, const void *pos_table, int64_t pos_rows,
                     const int64_t *row_index, int64_t x_rows,
                     const float *norm_weight, const float *norm_bias, float eps, int norm, void *out,
                     int64_t rows, int width, int dtype, void *stream);

/*
 * A gated RMS norm of each of `groups` equal parts of a row:
 *     PA_GATE_SIGMOID_LAST   out = o / rms(o) * weight * sigmoid(gate)
 *     PA_GATE_SILU_FIRST     z = o * silu(gate), out = z / rms(z) * weight
 *     PA_GATE_SILU_LAST      out = o / rms(o) * weight * silu(gate)
 *     PA_GATE_NONE           out = o / rms(o) * weight                (gate NULL)
 * gate and out rows are gate_stride and out_stride elements apart; weight : float[width].
 */
int pa_rms_gate(const void *o, const void *gate, int64_t gate_stride, const float *weight, float eps, void *out,
                int64_t out_stride, int64_t rows, int width, int groups, int gate_mode, int dtype, void *stream);

/* out = cap * tanh(x / cap), n elements of dtype to float. */
int pa_softcap(const void *x, float *out, int64_t n, float cap, int dtype, void *stream);

/*
 * out = act(gate) * up, rows of `width` elements at strides of their own.  With ids, row r's factor is row ids[r] of
 * `up`, a table of up_rows rows (a per-token input); ids out of range give zeros.
 */
int pa_glu(const void *gate, int64_t gate_stride, const void *up, int64_t up_stride, const int64_t *ids,
           int64_t up_rows, void *out, int64_t rows, int width, int act, int dtype, void *stream);

/* out = act(x + bias), rows of `width` elements at x_stride; bias : float[width] or NULL. */
int pa_bias_act(const void *x, int64_t x_stride, const float *bias, void *out, int64_t rows, int width, int act, int dtype,
                void *stream);

/*
 * out[row][h][0:vdim] = scale * o[row][h][0:vdim] * sigmoid(gate[row][h]): the gate of each head behind attention, and the
 * step from attention's padded rows (d) to packed ones (vdim), out_stride elements apart.  gate NULL: without it.
 */
int pa_head_gate(const void *o, const void *gate, int64_t gate_stride, float scale, void *out, int64_t out_stride,
                 int64_t rows, int heads, int d, int vdim, int dtype, void *stream);

/*
 * From joint projections to attention's operands: row = [q heads | k heads | v heads | anything].
 *   0. plus bias (float[channels], only without a convolution), when given;
 *   1. causal convolution over time per channel: y_t = sum_j w[j] u_(t - taps + 1 + j), the rows before a portion from
 *      conv_state (the last taps - 1 projected rows of the sequence, updated by the call);
 *      then, with q_norm and k_norm (float[dim]), q and k divided by sqrt(mean over dim of the square + eps) and times
 *      these weights;
 *   2. q, k: the pair (2i, 2i+1) of the first rot_dims dimensions turns by the angle whose (cos, sin) is
 *      rope[position][i];
 *   3. q, k: with unit_norm, divided by sqrt(mean over dim of the square + eps); q also times q_scale;
 *   4. v: as v_mode says; v_lambda is one float on the device;
 *   5. q to q_out, k and v to the pool at slots[row] (skipped when out of range), all in heads of pool_dim elements,
 *      the rest of a head zeros.
 *   conv_weight : float[taps][channels], channels = (Hq + Hkv) dim + Hkv vdim; taps <= 8 (1: no convolution)
 *   conv_state  : [state_rows][taps - 1][channels] of dtype, sequence b's at state_slots[b] (negative: zeros, unsaved)
 *   rope        : float[rope_rows][rot_dims / 2][2]
 *   tiles       : int32[n_tiles][2] = (sequence, first row inside its portion), every portion covered in steps of
 *                 PA_QKV_TILE_ROWS from row 0; NULL with n_tiles = batch: one row per sequence
 *   v_first     : [n_rows][Hkv * vdim] of dtype
 */
int pa_qkv_conv_append(const void *u, int64_t u_stride, int64_t n_rows, const float *bias, const float *conv_weight, int taps,
                       void *conv_state, int64_t state_rows, const float *rope, int64_t rope_rows, int rot_dims,
                       const int32_t *ctx_lens, const int32_t *q_lens, const int32_t *q_starts,
                       const int32_t *state_slots, const int32_t *tiles, int n_tiles, int batch,
                       const int64_t *slots, int64_t total_slots, void *q_out, void *k_cache, void *v_cache,
                       void *v_first, const float *v_lambda, int v_mode, const float *q_norm, const float *k_norm,
                       int num_q_heads, int num_kv_heads, int dim, int vdim, int pool_dim, int unit_norm, float eps,
                       float q_scale, int dtype, void *stream);

/*
 * Lightning attention: per head S_t = decay S_(t-1) + k_t v_t^T and o_t = S_t^T q_t, with q, k and v the silu of a
 * projection row [q heads | k heads | v heads | anything].
 *   state        : float[state_rows][heads][pad16(dim)][pad16(vdim)], zero-filled once (pa_lightning_state_floats gives
 *                  the floats per head); sequence b's at state_slots[b] (negative: starts empty, unsaved)
 *   decay_powers : float[heads][65], the powers 0 .. 64 of each head's decay
 *   out          : [n_rows][heads * vdim] of dtype
 *   dim <= 256, any vdim
 * pa_lightning_recurrent walks a portion token by token (decode steps; 32-bit prompts).  pa_lightning_chunked
 * (PA_BF16) multiplies 64 rows at a time on the matrix cores, with the 32-bit factors split into two bf16 terms; given
 * a workspace it cuts long portions of small batches into segments that run at the same time.  max_q_len: at least
 * the longest portion.
 */
size_t pa_lightning_state_floats(int dim, int vdim);
int pa_lightning_recurrent(const void *u, int64_t u_stride, int64_t n_rows, float *state, int64_t state_rows,
                           const float *decay_powers, const int32_t *ctx_lens, const int32_t *q_lens,
                           const int32_t *q_starts, const int32_t *state_slots, int batch, void *out,
                           int num_heads, int dim, int vdim, int dtype, void *stream);
size_t pa_lightning_workspace_bytes(int batch, int num_heads, int dim, int vdim, int max_q_len);
int pa_lightning_chunked(const void *u, int64_t u_stride, int64_t n_rows, float *state, int64_t state_rows,
                         const float *decay_powers, const int32_t *ctx_lens, const int32_t *q_lens,
                         const int32_t *q_starts, const int32_t *state_slots, int batch, int max_q_len,
                         void *out, int num_heads, int dim, int vdim, int dtype, void *workspace,
                         size_t workspace_bytes, void *stream);

/*
 * A causal convolution over time per channel, y_t = act(bias + sum_j w[j] u_(t - taps + 1 + j)), with the rows before a
 * portion from conv_state (the last taps - 1 input rows of the sequence, updated by the call).
 *   weight : float[taps][channels], bias : float[channels] or NULL;  taps <= 8;  act : PA_ACT_NONE or PA_ACT_SILU
 *   conv_state, tiles, n_tiles : as in pa_qkv_conv_append;  out : [n_rows][channels]
 */
int pa_short_conv(const void *u, int64_t u_stride, int64_t n_rows, const float *weight, const float *bias, int taps,
                  int act, void *conv_state, int64_t state_rows, const int32_t *ctx_lens, const int32_t *q_lens,
                  const int32_t *q_starts, const int32_t *state_slots, const int32_t *tiles, int n_tiles, int batch,
                  void *out, int channels, int dtype, void *stream);

/*
 * Linear recurrences with a decay and an input weight per token and head.  Per head (q and k of head h are those of
 * group h / heads_per_group):
 *   PA_GL_SSD    dt = softplus(gate_a + head_a);  S_t = exp(-head_b dt) S_(t-1) + dt k_t v_t^T;
 *                o_t = S_t^T q_t + head_c v_t                          (Mamba-2: q = C, k = B, v = x, head_b = exp(A_log))
 *   PA_GL_MLSTM  i = cap tanh((gate_a + head_a) / cap);  f = logsigmoid(cap tanh((gate_b + head_b) / cap));
 *                m_t = max(f + m_(t-1), i), m_0 = 0;  S_t = exp(f + m_(t-1) - m_t) S_(t-1) + exp(i - m_t) k_t v_t^T;
 *                n_t likewise with k alone;  o_t = q_scale S_t^T q_t / (max(|q_scale n_t . q_t|, exp(-m_t)) + den_eps)
 *   q, k, v       : rows of dtype at strides of their own (column slices of a projection)
 *   gate_a, gate_b: gate logits [row][head] of dtype, gate_stride elements between rows
 *   state         : float[state_rows][heads][pa_gated_linear_state_floats(kind, dim, vdim)], zero-filled once; sequence
 *                   b's at state_slots[b] (negative: starts empty, unsaved)
 *   out           : [n_rows][heads * vdim] of dtype;  dim <= 256, any vdim
 * Single rows (q_lens NULL), PA_F32 and rows that are not whole 8-byte vectors run token by token; PA_BF16 portions in
 * chunks of 64 rows on the matrix cores, with the 32-bit factors split into two bf16 terms, and, given a workspace, in
 * segments that run at the same time when there are few sequences.  max_q_len: at least the longest portion.
 */
size_t pa_gated_linear_state_floats(int kind, int dim, int vdim);
size_t pa_gated_linear_workspace_bytes(int batch, int num_heads, int dim, int vdim, int max_q_len);
int pa_gated_linear(int kind, const void *q, int64_t q_stride, const void *k, int64_t k_stride, const void *v,
                    int64_t v_stride, int heads_per_group, const void *gate_a, const void *gate_b, int64_t gate_stride,
                    const float *head_a, const float *head_b, const float *head_c, float cap, float q_scale,
                    float den_eps, int64_t n_rows, float *state, int64_t state_rows, const int32_t *ctx_lens,
                    const int32_t *q_lens, const int32_t *q_starts, const int32_t *state_slots, int batch,
                    int max_q_len, void *out, int num_heads, int dim, int vdim, int dtype, void *workspace,
                    size_t workspace_bytes, void *stream);

/* out = x w^T with 32-bit sums and results, for few outputs: x [rows] at x_stride, w [n][k], out float[rows][n]. */
int pa_narrow_linear(const void *x, int64_t x_stride, const void *w, float *out, int64_t rows, int n, int k, int dtype,
                     void *stream);

/*
 * The gated delta rule.  Per head, with q and k of group h / heads_per_group divided by sqrt(sum of squares + 1e-6) and q also
 * times q_scale:
 *     g_t = exp(-decay_rate softplus(decay_logit + decay_bias));  beta_t = sigmoid(beta_logit);
 *     S <- g_t S_(t-1);  u = beta_t (v_t - S^T k_t);  S_t = S + k_t u^T;  o_t = S_t^T q_t
 * Tensors, state (float[state_rows][heads][pad16(dim)][pad16(vdim)]) and kernels as in pa_gated_linear; 16-bit portions are
 * multiplied in chunks of 64 rows when the workspace holds pa_delta_workspace_bytes, else they run token by token.
 */
size_t pa_delta_workspace_bytes(int batch, int num_heads, int dim, int vdim, int max_q_len);
int pa_delta(const void *q, int64_t q_stride, const void *k, int64_t k_stride, const void *v, int64_t v_stride,
             int heads_per_group, const void *decay_logits, const void *beta_logits, int64_t gate_stride,
             const float *decay_bias, const float *decay_rate, float q_scale, int64_t n_rows, float *state,
             int64_t state_rows, const int32_t *ctx_lens, const int32_t *q_lens, const int32_t *q_starts,
             const int32_t *state_slots, int batch, int max_q_len, void *out, int num_heads, int dim, int vdim, int dtype,
             void *workspace, size_t workspace_bytes, void *stream);

/*
 * Residual streams (hyper-connections), one row at a time: x[row][s], s < streams <= 16.
 *     x_t = table[ids[row]] for every t             when ids is given; else, when y is given,
 *     x_t = sum_s between[s][t] x_s + into[t] y     (all from the old streams; written back unless `sum` is given)
 *     z = sum_t sum_weight[t] x_t                   (NULL: ones)
 *     out = z / rms(z) * norm_weight;  sum = z      whichever is given
 * With mix_weight (float[rows][mix_stride]) y is the weighted sum over i < mix of y[row * mix + i], plus y_extra[row] under
 * weight mix and y_self[row] under weight mix + 1 where given; rows under a weight of exactly 0 are not read.
 *   x : float[rows][streams][width];  y, y_extra, y_self, table, out : dtype;  sum : float[rows][width];  width <= 16384
 */
int pa_hyper_norm(float *x, const void *y, const float *mix_weight, int mix, int mix_stride, const void *y_extra,
                  const void *y_self, const float *between, const float *into, const int64_t *ids, const void *table,
                  int64_t table_rows, const float *sum_weight, const float *norm_weight, float eps, void *out, float *sum,
                  int64_t rows, int streams, int width, int dtype, void *stream);

/*
 * Latent attention's operands from rows [heads of dim + rot_dim | rank | rot_dim]: q_out gets every head times q_scale with
 * its last rot_dim elements turned (pairs 2i, 2i + 1 by rope[position][i]), zeros up to q_dim; the pool's row of the token
 * is [rank elements / rms * norm_weight | last rot_dim elements turned | zeros] of pool_row elements.  Portions, tiles and
 * slots as in pa_qkv_conv_append.
 * pa_latent_gather: out[r] = pool row slots[r], zeros for slots out of range.
 */
int pa_latent_append(const void *u, int64_t u_stride, int64_t n_rows, const float *norm_weight, float eps, const float *rope,
                     int64_t rope_rows, const int32_t *ctx_lens, const int32_t *q_lens, const int32_t *q_starts,
                     const int32_t *tiles, int n_tiles, int batch, const int64_t *slots, int64_t total_slots, void *q_out,
                     void *pool, int num_heads, int dim, int rot_dim, int rank, int q_dim, int pool_row, float q_scale,
                     int dtype, void *stream);
int pa_latent_gather(const void *pool, const int64_t *slots, int64_t total_slots, void *out, int64_t rows, int pool_row,
                     int dtype, void *stream);

/*
 * Paged attention with score terms.  For the row at position i, over the visible keys j <= i (window > 0: i - j < window):
 *     score_j = softcap tanh(scale q . k_j / softcap) + bias[h][min(i - j, bias_n - 1)]     (softcap 0, bias NULL: without)
 *     out = sum_j e^score_j v_j / (sum_j e^score_j + e^sink[h])                              (sink NULL: without)
 * A query is n1 elements of q1 followed by n2 of q2, head h of row r at r * q_row + h * q_head.  k_cache, v_cache: pool
 * rows [slot][kv head][k_dim], [slot][kv head][v_dim], of which the first n1 + n2 and vdim count; v_cache may point into
 * k_cache's rows.  out : [n_rows][heads][vdim].  Missing blocks read as zero rows.  16-bit decode steps (q_lens NULL) with
 * a workspace spread a sequence's keys over the device.
 */
size_t pa_scored_workspace_bytes(int batch, int num_q_heads, int num_kv_heads, int key_size, int vdim, int one_tensor,
                                 int64_t max_keys, int window);
int pa_scored_attention(const void *q1, int64_t q1_row, int64_t q1_head, int n1, const void *q2, int64_t q2_row,
                        int64_t q2_head, int n2, const void *k_cache, int k_dim, const void *v_cache, int v_dim, int vdim,
                        const int32_t *block_tables, int64_t bt_stride, int block_size, int64_t num_blocks,
                        const int32_t *ctx_lens, const int32_t *q_lens, const int32_t *q_starts, int64_t n_rows, int batch,
                        int max_q_len, int num_q_heads, int num_kv_heads, float scale, int window, float softcap,
                        const float *bias, int bias_n, const float *sink, void *out, int dtype, void *workspace,
                        size_t workspace_bytes, void *stream);

/*
 * Paged attention whose heads' weights are mixed before they meet the values.  For the row at position i, over the visible
 * keys j <= i:
 *     s_h(j) = scale q_h . k_j - bias_size[h] ln(1 + bias_rate[h] (i - j))        (bias_size, bias_rate NULL: without)
 *     p_h = softmax of s_h;  w_h(j) = sum_g talk[h][g] p_g(j);  out_h = sum_j w_h(j) v_j      (v of h's own kv head)
 * q: head h of row r at r * q_row + h * q_head, dim elements; pools as in pa_scored_attention.  bias_size, bias_rate :
 * float[Hq]; talk : float[Hq][Hq]; out : [n_rows][Hq][vdim].  Hq <= 128, dim and vdim <= 256.  The workspace
 * (pa_talking_workspace_bytes, decode: q_lens NULL; max_keys = bt_stride * block_size) holds the sums of every row and head and,
 * for 16-bit decode steps, the scores and the parts of the output that a sequence's pieces leave; less than that but enough
 * for the sums runs on the vector units.
 */
size_t pa_talking_workspace_bytes(int64_t n_rows, int batch, int num_q_heads, int num_kv_heads, int vdim, int64_t max_keys, int decode);
int pa_talking_attention(const void *q, int64_t q_row, int64_t q_head, int dim, const void *k_cache, int k_dim, const void *v_cache,
                         int v_dim, int vdim, const int32_t *block_tables, int64_t bt_stride, int block_size, int64_t num_blocks,
                         const int32_t *ctx_lens, const int32_t *q_lens, const int32_t *q_starts, int64_t n_rows, int batch,
                         int max_q_len, int num_q_heads, int num_kv_heads, float scale, const float *bias_size,
                         const float *bias_rate, const float *talk, void *out, int dtype, void *workspace,
                         size_t workspace_bytes, void *stream);

/*
 * Linear attention with a forget gate per channel that also decides what is written.  Per head and channel, with act one of
 * PA_ACT_NONE and PA_ACT_SILU:
 *     f_t = lower + (1 - lower) sigmoid(forget_t + f_bias);  S_t = diag(f_t) S_(t-1) + (1 - f_t) v_t^T;  o_t = S_t^T act(q_t)
 *   q, forget, v : rows of dtype at strides of their own;  f_bias (or NULL), lower : float[heads * dim]
 *   state        : float[state_rows][heads][pad16(dim)][pad16(vdim)]; slots, portions and kernels as in pa_gated_linear
 *   out          : [n_rows][heads * vdim] of dtype;  dim <= 256, any vdim
 */
size_t pa_channel_linear_workspace_bytes(int batch, int num_heads, int dim, int vdim, int max_q_len);
int pa_channel_linear(const void *q, int64_t q_stride, int q_act, const void *forget, int64_t f_stride, const float *f_bias,
                      const float *lower, const void *v, int64_t v_stride, int64_t n_rows, float *state, int64_t state_rows,
                      const int32_t *ctx_lens, const int32_t *q_lens, const int32_t *q_starts, const int32_t *state_slots,
                      int batch, int max_q_len, void *out, int num_heads, int dim, int vdim, int dtype, void *workspace,
                      size_t workspace_bytes, void *stream);

/*
 * Mixture of experts.  pa_moe_choose, per row over the experts and, behind them, `identity` identity experts (which hand on the
 * row's own input): scores s = sigmoid(logits) or their softmax; choice scores s + correction (NULL: s).  Of `groups`
 * equal groups of neighbours the `keep` with the largest sums of their group_top (1 or 2) largest choice scores stay; of
 * their experts the `top` with the largest choice scores are chosen (the lowest number first on ties).  ids int32[rows][top],
 * -1 for an identity expert; weights float[rows][top + 1], with identity experts [top + 2]: the chosen s (renormalize: over
 * their sum + 1e-20; 0 in the place of an identity expert), the shared expert's sigmoid(logits[experts]), 1 or 0 as
 * `shared` says, and the sum of the chosen identity experts' s.  top <= 64, experts + identity <= 1024.  And per expert
 * (identity ones included) counts int32[] and lists int32[][rows]: its items (row * top + place) in order.  (Scores that
 * are NaN are not chosen: id -1.)  The workspace is for experts + identity and needs no initial contents.
 * pa_moe_product: for every listed item, out[item] = W_e x[item / items_per_row], or with glu
 * silu(G_e x) * (U_e x) where an expert's weight rows are the n rows of G followed by the n rows of U.
 *   w : [experts][w_rows][w_stride] of dtype, rows zero past k.  The matrix-core kernels want w_stride % 64 == 0,
 *   k % 8 == 0, n % 4 == 0 and 16-byte aligned tensors; anything else runs on the vector units.
 */
size_t pa_moe_workspace_bytes(int64_t rows, int experts, int top);
int pa_moe_choose(const float *logits, int64_t logits_stride, int64_t rows, int experts, int identity, int top, int groups,
                  int keep, int shared, int scores, int group_top, int renormalize, const float *correction, int32_t *ids,
                  float *weights, int32_t *counts, int32_t *lists, void *workspace, size_t workspace_bytes, void *stream);
int pa_moe_product(const void *x, int64_t x_stride, int items_per_row, const void *w, int64_t w_rows, int w_stride, int k,
                   const int32_t *counts, const int32_t *lists, int64_t rows, int top, int experts, int glu, void *out,
                   int n, int dtype, void *stream);

#ifdef __cplusplus
}
#endif
#endif /* PAGED_ATTN_H */
