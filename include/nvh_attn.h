/*
 * nvh_attn.h — C ABI of the MI355X (gfx950) paged-attention backend for nano-vllm.
 *
 * This is the drop-in boundary for `--attn-backend hip`: the entry points below are exactly
 * what a reference-side binding (ctypes) calls from
 * nanovllm/layers/attention.py's `Attention.forward`.  Plain C, raw device pointers and sizes,
 * no torch / pybind types.  One process per GPU, single caller thread per process.
 *
 * Contract:
 *   - The caller owns ALL memory, including the decode workspace.  The library allocates nothing,
 *     frees nothing and keeps no state besides a thread-local error string.
 *   - Every call only enqueues kernels on `stream` (a hipStream_t; NULL = default stream).  No host
 *     synchronisation, no host reads of device data, grid sizes are functions of the static
 *     arguments only -> every call is legal inside HIP-graph capture
 *     (nanovllm/engine/model_runner.py:316-370 captures the decode forward).
 *   - Return 0 on success; a negative NVH_E_* code for rejected arguments; a positive hipError_t
 *     for a failed launch.  nvh_last_error() gives the message.  Nothing throws across the ABI.
 *   - K/V cache layout is the reference's: [num_blocks, block_size, num_kv_heads, head_dim],
 *     contiguous (model_runner.py:144-145, asserts attention.py:51-54).  All cache offsets are
 *     64-bit inside the kernels.
 *   - Element type of q/k/v/caches: bf16 (NVH_BF16), the reference's runtime dtype
 *     (model_runner.py:35).  Outputs are bf16, or fp32 (NVH_F32) for pre-rounding parity checks.
 *   - softmax scale is passed explicitly and must be head_dim**-0.5 to match the reference's
 *     flash / sdpa backends (attention.py:96,101).
 */
#ifndef NVH_ATTN_H
#define NVH_ATTN_H

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

#define NVH_VERSION 206          /* major*100 + minor; 201: nvh_allreduce_status; 202: nvh_linear_desc.prefetch; 203: NVH_DECODE_CHUNKED_P256; 204: nvh_qkv_rope_attend; 205: nvh_prefill_varlen_pv16; 206: nvh_linear_desc.glu_*, nvh_rglru_*, nvh_latent_* */

/* dtype codes */
#define NVH_BF16 0
#define NVH_F32  1

/* argument errors (negative so they never collide with hipError_t) */
#define NVH_E_DTYPE      (-1)    /* unsupported element type */
#define NVH_E_SHAPE      (-2)    /* unsupported head_dim / group size / block_size */
#define NVH_E_STRIDE     (-3)    /* stride not a multiple of 8 elements (16-byte vector access) */
#define NVH_E_WORKSPACE  (-4)    /* workspace too small */
#define NVH_E_NULL       (-5)    /* required pointer is NULL */
#define NVH_E_ALIGN      (-6)    /* pointer not 16-byte aligned */

int nvh_version(void);
const char* nvh_last_error(void);

/*
 * Scatter new K/V rows into the paged cache.
 * Replaces: store_kvcache + store_kvcache_kernel, nanovllm/layers/attention.py:19-55
 *           (slot < 0 rows are skipped, as nanovllm/layers/attention_triton.py:29-31 does for -1).
 *   k, v           [n_tokens, kvh, hd]; inner two dims contiguous, row strides in ELEMENTS
 *                  (v is a strided view of the fused qkv projection, models/qwen3.py:104-106)
 *   k_cache/v_cache [num_blocks, block_size, kvh, hd] contiguous; row `slot` = slot*kvh*hd elements
 *   slot_mapping   int32 [n_tokens], slot = block_id*block_size + offset (model_runner.py:212-221,254-258)
 * n_tokens == 0 is a no-op.
 */
int nvh_store_kvcache(const void* k, const void* v, void* k_cache, void* v_cache,
                      const int32_t* slot_mapping, int n_tokens, int kvh, int hd,
                      int64_t k_row_stride, int64_t v_row_stride, int dtype, void* stream);

/*
 * Bytes of caller-owned scratch nvh_paged_decode needs; a pure function of the static shapes so it can be
 * allocated once before graph capture.  Layout: a fixed 64 KiB header of arrival tickets (one uint32 per
 * (sequence, kv head), each on a 128-byte line of its own: 512 pairs can be split over several workgroups, far more than the
 * device has CUs for), 8 KiB of counters for nvh_qkv_rope_attend's hand-off (ready / done per kv head, one per line; a status word),
 * then the partial records of the context chunks (each padded to a 256-byte boundary).  The caller ZERO-FILLS the buffer once
 * (hipMemset / torch.zeros); every launch returns its tickets to zero, so the buffer is reusable across calls,
 * shapes and graph replays without further clearing.  ONE launch at a time per workspace: calls that may run concurrently
 * (different streams) need a workspace each; a launch that was aborted mid-flight leaves the tickets undefined (zero-fill again).
 */
size_t nvh_paged_decode_workspace(int batch, int h, int hd, int max_blocks, int block_size);

/*
 * Decode: one query token per sequence attends its whole paged context.
 * Replaces: flash_attn_with_kvcache(q.unsqueeze(1), k_cache, v_cache, cache_seqlens=context_lens,
 *           block_table=block_tables, softmax_scale, causal=True), nanovllm/layers/attention.py:99-101
 *           (oracle body nanovllm/layers/attention_sdpa.py:122-182).
 *   out            [batch, h, hd]  (out_dtype NVH_BF16 or NVH_F32), contiguous
 *   q              [batch, h, hd], contiguous per row; q_row_stride in elements
 *   block_tables   int32 [batch, max_blocks], row stride bt_row_stride (elements); entries at or past
 *                  ceil(ctx/block_size) are never dereferenced (they are -1 in eager mode and 0 under
 *                  graph replay, model_runner.py:160-169,299)
 *   context_lens   int32 [batch]; 0 -> the row's output is zeros (graph padding rows)
 *   h % kvh == 0, h/kvh <= 16, hd in {64, 128},
 *   block_size a multiple of 64.
 */
int nvh_paged_decode(void* out, const void* q, const void* k_cache, const void* v_cache,
                     const int32_t* block_tables, const int32_t* context_lens,
                     int batch, int h, int kvh, int hd, int block_size, int max_blocks,
                     int64_t q_row_stride, int64_t bt_row_stride, float scale,
                     int dtype, int out_dtype, void* workspace, size_t workspace_bytes, void* stream);

/*
 * The same call through a chosen formulation of the decode kernel (tests and A/B measurements; nvh_paged_decode always runs
 * NVH_DECODE_CHUNKED with waves = chunks = 0).  All variants compute the same function and are held to the same parity bar:
 *   NVH_DECODE_CHUNKED     one launch: MFMA tiles over the GQA group, split-KV passes dealt to `chunks` workgroups per
 *                          (sequence, kv head), last-arriver combine.  waves per workgroup: 4 or 8; 0 = the default (8 at hd 64, 4 at hd 128).
 *                          chunks: 0 = one wave of workgroups over the device's CUs, > 0 = that many (clamped to the passes).
 *                          hd 64: passes of 256 tokens, or of 128 where a pair is split over 3-5 workgroups (few passes per workgroup:
 *                          the finer passes balance the workgroups better; measured -2.5 % on average there, +1..12 % with more chunks)
 *   NVH_DECODE_CHUNKED_P128 / _P256 / _P64  the chunked kernel with the pass size forced: hd 64 takes 128 or 256 (16- / 32-token wave tiles),
 *                          hd 128 takes 128 or 64 (four waves x 32- / 16-token tiles; the default picks 64 where a pair is split over at most
 *                          8 workgroups: -5 % at Qwen2-7B's per-rank shape 7/1/128, bs 32); a size the head_dim does not have is ignored
 *   NVH_DECODE_SPLIT_MFMA  the single-pass MFMA split kernel + a combine launch (flash-decoding in two launches).
 *   NVH_DECODE_SPLIT_VALU  north_star's literal form: VALU dot products with wavefront-level (DPP / permlane) max and sum
 *                          reductions, no MFMA; groups of at most 8 query heads per kv head; + the combine launch.
 */
enum { NVH_DECODE_CHUNKED = 0, NVH_DECODE_SPLIT_MFMA = 1, NVH_DECODE_SPLIT_VALU = 2, NVH_DECODE_CHUNKED_P128 = 3, NVH_DECODE_CHUNKED_P256 = 4, NVH_DECODE_CHUNKED_P64 = 5 };
int nvh_paged_decode_variant(int variant, int waves, int chunks, void* out, const void* q, const void* k_cache, const void* v_cache,
                             const int32_t* block_tables, const int32_t* context_lens,
                             int batch, int h, int kvh, int hd, int block_size, int max_blocks,
                             int64_t q_row_stride, int64_t bt_row_stride, float scale,
                             int dtype, int out_dtype, void* workspace, size_t workspace_bytes, void* stream);

/*
 * nvh_paged_decode that ALSO writes the bf16 result in MFMA-fragment order (out_packed: [ceil(batch/16)][h*hd/32][64][8],
 * nvh_pack_index(row = sequence, col = head*hd + dim, cols = h*hd)) for a following nvh_linear_small_m_ex with x_packed = 1
 * (the output projection, models/qwen3.py:118).  Same arguments otherwise; `out` is still written.
 */
int nvh_paged_decode_packed(void* out, void* out_packed, const void* q, const void* k_cache, const void* v_cache,
                            const int32_t* block_tables, const int32_t* context_lens,
                            int batch, int h, int kvh, int hd, int block_size, int max_blocks,
                            int64_t q_row_stride, int64_t bt_row_stride, float scale,
                            int dtype, int out_dtype, void* workspace, size_t workspace_bytes, void* stream);

/*
 * Fused decode step for one layer: store this step's K/V row of every sequence, then attend.
 * Replaces the pair of calls at nanovllm/layers/attention.py:84-86 and :99-101 with one launch
 * sequence; result identical to nvh_store_kvcache followed by nvh_paged_decode.
 *   k_new, v_new   [batch, kvh, hd] with row strides in elements; slot_mapping int32 [batch]
 */
int nvh_decode_step(void* out, const void* q, const void* k_new, const void* v_new,
                    void* k_cache, void* v_cache, const int32_t* slot_mapping,
                    const int32_t* block_tables, const int32_t* context_lens,
                    int batch, int h, int kvh, int hd, int block_size, int max_blocks,
                    int64_t q_row_stride, int64_t k_row_stride, int64_t v_row_stride,
                    int64_t bt_row_stride, float scale, int dtype, int out_dtype,
                    void* workspace, size_t workspace_bytes, void* stream);

/*
 * Prefill: packed variable-length causal attention.
 * Replaces: flash_attn_varlen_func(q, k, v, cu_seqlens_q/k, max_seqlen_q/k, softmax_scale,
 *           causal=True, block_table=...), nanovllm/layers/attention.py:93-96
 *           (oracle body nanovllm/layers/attention_sdpa.py:65-119).
 *   block_tables == NULL : k, v are the new tokens [total_k, kvh, hd] with row strides (elements).
 *   block_tables != NULL : k, v are the paged caches (prefix-cache prefill, attention.py:90-91);
 *                          k/v_row_stride are ignored; sequence i's keys are found through
 *                          block_tables[i, :]; block_size/max_blocks/bt_row_stride describe it.
 *   cu_seqlens_q/k int32 [batch+1] on device; max_seqlen_q bounds the launch grid (host int, as in
 *                  model_runner.py:204-207).  The causal mask is bottom-right aligned: query row r
 *                  of a sequence sees keys 0 .. r + (Sk - Sq)  (flash-attn semantics; equals the
 *                  oracle's top-left mask whenever Sq == Sk).
 *                  CONTRACT: max_seqlen_q / max_seqlen_k must bound every sequence in cu_seqlens_q/k (as the reference's
 *                  runner guarantees).  The library cannot check device data without a host sync; rows / keys beyond an
 *                  understated maximum are not processed (never an out-of-bounds access).
 *   out            [total_q, h, hd] contiguous, out_dtype NVH_BF16 or NVH_F32.
 */
int nvh_prefill_varlen(void* out, const void* q, const void* k, const void* v,
                       const int32_t* cu_seqlens_q, const int32_t* cu_seqlens_k,
                       const int32_t* block_tables, int batch, int max_seqlen_q, int max_seqlen_k,
                       int h, int kvh, int hd, int block_size, int max_blocks,
                       int64_t q_row_stride, int64_t k_row_stride, int64_t v_row_stride,
                       int64_t bt_row_stride, float scale, int dtype, int out_dtype, void* stream);

/*
 * The same call with the kernel chosen by the caller (tests and A/B measurements; nvh_prefill_varlen passes 0, 0):
 *   kernel       NVH_PREFILL_AUTO, NVH_PREFILL_TILED (64-row query tiles, K/V tiles double-buffered through LDS) or
 *                NVH_PREFILL_SHORT (one workgroup per (sequence, kv head), K/V resident in LDS: needs max_seqlen_q <=
 *                max_seqlen_k <= 128 and block_tables == NULL, otherwise an error)
 *                NVH_PREFILL_TILED_F16V (a MEASUREMENT variant, not a drop-in: block_tables must be NULL): `v` holds the values as IEEE fp16 rows,
 *                converted by the caller (same layout and strides); P is rounded to fp16 and P V runs as one fp16 MFMA per operand pair instead
 *                of the bf16 hi + lo pair.  Error 4.5e-4 on the reference goldens (hi + lo: 6e-6), |v| <= 65504 required; DESIGN.md section 12.2
 *   short_waves  waves per workgroup of the short-sequence kernel: 0 = auto, 8 or 16
 */
enum { NVH_PREFILL_AUTO = 0, NVH_PREFILL_TILED = 1, NVH_PREFILL_SHORT = 2, NVH_PREFILL_TILED_F16V = 3 };
int nvh_prefill_varlen_variant(int kernel, int short_waves, void* out, const void* q, const void* k, const void* v,
                               const int32_t* cu_seqlens_q, const int32_t* cu_seqlens_k,
                               const int32_t* block_tables, int batch, int max_seqlen_q, int max_seqlen_k,
                               int h, int kvh, int hd, int block_size, int max_blocks,
                               int64_t q_row_stride, int64_t k_row_stride, int64_t v_row_stride,
                               int64_t bt_row_stride, float scale, int dtype, int out_dtype, void* stream);

/* Helper of the NVH_PREFILL_TILED_F16V measurement form: bf16 rows [n_rows, row_elems] (row strides in elements) -> IEEE fp16 rows, exact for
 * 2^-24 <= |x| <= 65504 (larger finite magnitudes are clamped: the caller must know its V stays in range — nvh_prefill_varlen_pv16 below checks it).
 * 16-byte aligned rows, row_elems % 8 == 0. */
int nvh_bf16_rows_to_f16(void* out, const void* in, int n_rows, int row_elems, int64_t in_row_stride, int64_t out_row_stride, void* stream);

/*
 * nvh_prefill_varlen (block_tables == NULL) with P V on the fp16 matrix pipe — same arguments, same result within the parity bar, 1.2-1.4x faster from 1024
 * keys per sequence on (the tile loop is bound by vector-instruction issue and the bf16 hi + lo split of P is a third of it).
 * Replaces: flash_attn_varlen_func, nanovllm/layers/attention.py:93-96 (whose own P is a single bf16: 8 significant bits against the 11 used here).
 * Two launches, no host read, nothing to clear, capture-safe: V is converted to fp16 rows in `scratch` (exact for 2^-24 <= |v| <= 65504; smaller magnitudes
 * become 0) and every 64-row group gets a range flag (set when a finite value does not fit fp16); the attention kernel ORs the flags that cover a
 * sequence's rows and runs fp16 P x fp16 V for it, or — a flag set, or the sequence reaching past total_k — the exact bf16 hi + lo form on the caller's own
 * V rows, i.e. exactly nvh_prefill_varlen for that sequence.  Numerics of the fp16 form: P in [0, 1] rounded to 11 significant bits, products accumulated
 * in fp32: |error| <= 2^-12 * max|v| per output element, 4.5e-4 on the reference's golden vectors (N(0,1) values; hi + lo: 6e-6; bf16 OUTPUT rounding
 * alone: 2^-9 * |o|).  Shapes the short-sequence kernel takes (max_seqlen_q <= max_seqlen_k <= 128, >= 128 (sequence, kv head) pairs:
 * nvh_prefill_pv16_uses_scratch() == 0, scratch may be NULL) run ONE launch: at head_dim 64 and more than 64 keys each workgroup converts its resident
 * V images to fp16 in LDS, range check folded into the barrier that publishes them (a (sequence, kv head) pair out of range keeps hi + lo); otherwise
 * that kernel runs unchanged.
 *   total_k        rows of k / v (= cu_seqlens_k[batch] on the host)
 *   scratch        device memory of at least nvh_prefill_pv16_scratch_bytes(total_k, kvh, hd) bytes (flags: 4 * ceil(total_k / 64) rounded up to 256, then
 *                  total_k*kvh*hd*2), 16-byte aligned, owned by the caller, not shared with a call in flight on another stream
 */
size_t nvh_prefill_pv16_scratch_bytes(int total_k, int kvh, int hd);
int nvh_prefill_pv16_uses_scratch(int batch, int max_seqlen_q, int max_seqlen_k, int kvh, int hd);
int nvh_prefill_varlen_pv16(void* out, const void* q, const void* k, const void* v,
                            const int32_t* cu_seqlens_q, const int32_t* cu_seqlens_k, int batch, int max_seqlen_q, int max_seqlen_k, int total_k,
                            int h, int kvh, int hd, int64_t q_row_stride, int64_t k_row_stride, int64_t v_row_stride,
                            float scale, int dtype, int out_dtype, void* scratch, size_t scratch_bytes, void* stream);

/*
 * "Next" row: the step immediately before attention, fused into one launch.
 * (optional per-head RMSNorm ->) neox RoPE on q and k IN PLACE inside the fused qkv projection output, then
 * k (rotated) and v rows are stored to the paged cache.
 * Replaces: q_norm/k_norm (nanovllm/models/qwen3.py:108-114, layers/layernorm.py:17-27), rotary_emb
 *           (layers/rotary_embedding.py:39-55) and store_kvcache (layers/attention.py:84-86).
 *   qkv            [n_tokens, (h + 2*kvh) * hd] bf16, row stride qkv_row_stride (elements): q heads | k heads | v heads
 *   positions      int64 [n_tokens]; cos_sin fp32 [max_position, hd] = cos(0..hd/2) | sin(0..hd/2)
 *                  (the reference's cos_sin_cache, rotary_embedding.py:29-36)
 *   q_norm_w/k_norm_w  bf16 [hd] or NULL (both or neither); eps as in RMSNorm
 *   k_cache/v_cache/slot_mapping  as nvh_store_kvcache; NULL caches or slot < 0 -> no store for that row
 */
int nvh_rope_store(void* qkv, const int64_t* positions, const float* cos_sin,
                   const void* q_norm_w, const void* k_norm_w, float eps,
                   void* k_cache, void* v_cache, const int32_t* slot_mapping,
                   int n_tokens, int h, int kvh, int hd, int64_t qkv_row_stride, int dtype, void* stream);

/*
 * Engine widening (not part of the attention parity bar): the row-wise elementwise ops either side of the attention
 * block, one launch each instead of 5-6 eager launches per layer.
 *   nvh_add_rmsnorm  RMSNorm.forward(x[, residual]), nanovllm/layers/layernorm.py:17-50: if `residual` is non-NULL it is
 *                    updated in place to bf16(x + residual) and the norm is taken of the fp32 sum; out = norm * weight.
 *                    x/out/residual [n_rows, hidden] bf16 with row strides in elements; hidden % 8 == 0, hidden <= 8192.
 *   nvh_silu_mul     SiluAndMul.forward, nanovllm/layers/activation.py:11-14: out[:, i] = silu(gu[:, i]) * gu[:, inter + i].
 */
int nvh_add_rmsnorm(void* out, const void* x, void* residual, const void* weight, float eps, int n_rows, int hidden,
                    int64_t x_row_stride, int64_t out_row_stride, int64_t residual_row_stride, int dtype, void* stream);
int nvh_silu_mul(void* out, const void* gate_up, int n_rows, int inter, int64_t gate_up_row_stride, int64_t out_row_stride,
                 int dtype, void* stream);
/*   nvh_argmax_rows  greedy sampling (temperature 0; nanovllm/layers/sampler.py, bench_my.py:31): out[i] = argmax_j x[i, j],
 *                    int64, ties -> lowest index; x [n_rows, n] bf16, 16-byte aligned rows (row stride % 8 == 0). */
int nvh_argmax_rows(int64_t* out, const void* x, int n_rows, int n, int64_t x_row_stride, int dtype, void* stream);
/*   nvh_greedy_advance  the same arg-max fused with the host work between two decode steps, done on the device so a step is
 *                    pure graph replay: append the token (engine/scheduler.py:99-110) and rebuild next step's decode metadata
 *                    (engine/model_runner.py:244-269): tokens_log[row_steps[r], r] = tok; row_steps[r]++; input_ids[r] = tok;
 *                    positions[r]++; context_lens[r]++; slot_mapping[r] = block_tables[r, (ctx-1)/bs]*bs + (ctx-1)%bs with the
 *                    new ctx.  Rows whose context_lens is 0 (graph padding) are left untouched. */
int nvh_greedy_advance(const void* logits, int n_rows, int n, int64_t logits_row_stride,
                       int64_t* input_ids, int64_t* positions, int32_t* context_lens, int32_t* slot_mapping,
                       const int32_t* block_tables, int64_t bt_row_stride, int block_size,
                       int64_t* tokens_log, int64_t log_row_stride, int64_t* row_steps, int dtype, void* stream);

/*
 * Engine widening: weight-streaming linear layer for decode-sized batches, out = x . W^T (+ bias), m <= 64 rows.
 * Replaces F.linear in nanovllm/layers/linear.py:55-190 at decode (the hipBLASLt path stays for larger m).
 *   x [m, k] bf16 (row stride in elements); w [n, k] bf16 contiguous (nn.Linear layout); bias [n] bf16 or NULL
 *   silu_inter == 0 : out [m, n] = x w^T + bias
 *   silu_inter  > 0 : n == 2*silu_inter, rows [0, inter) of w are gate_proj and [inter, 2*inter) up_proj
 *                     (MergedColumnParallelLinear, linear.py:90-111); out [m, inter] = SiLU(x gate^T) * (x up^T), i.e. the
 *                     projection and layers/activation.py:11-14 in one launch; bias must be NULL.
 *   k % 64 == 0, n % 16 == 0 (and inter % 16 == 0).
 */
int nvh_linear_small_m(void* out, const void* x, const void* w, const void* bias, int m, int n, int k, int silu_inter,
                       int64_t x_row_stride, int64_t out_row_stride, int dtype, void* stream);

/*
 * The same weight-streaming product with the neighbouring row-wise ops of a decoder layer fused in, so that a decode
 * layer is 6 launches (qkv, attention split, attention combine, o_proj, gate_up, down) instead of 10:
 *   norm_weight != NULL : prologue x := RMSNorm(x) * norm_weight   (RMSNorm.rms_forward, nanovllm/layers/layernorm.py:17-27)
 *   norm_folded != 0    : the same norm with its weight already multiplied into w by the caller (w := w * diag(norm_weight));
 *                         sum(x^2) is taken inside the K loop and rows are scaled by rsqrt(mean(x^2) + norm_eps) in the epilogue
 *                         (same algebra, without re-rounding the normalised activations to bf16); norm_weight must be NULL
 *   epilogue NVH_EPI_NONE          out [m, n] = product + bias
 *            NVH_EPI_SILU_MUL      as nvh_linear_small_m with silu_inter
 *            NVH_EPI_RESIDUAL_ADD  out is the residual stream [m, n]: out += product, in place (the add of
 *                                  add_rms_forward, layernorm.py:35-36, done by the producing GEMM instead of the consuming norm)
 *            NVH_EPI_ROPE_STORE    n == (h + 2*kvh) * hd (fused qkv projection, models/qwen3.py:104-106): + bias, neox RoPE on
 *                                  the q and k heads, q -> out [m, h*hd]; k and v rows -> k_cache / v_cache at slot_mapping[row]
 *                                  (slot < 0: skipped).  Same arithmetic and rounding points as nvh_rope_store; no q/k norm.
 */
#define NVH_EPI_NONE          0
#define NVH_EPI_SILU_MUL      1
#define NVH_EPI_RESIDUAL_ADD  2
#define NVH_EPI_ROPE_STORE    3
typedef struct nvh_linear_desc {
    void* out;
    const void* x;
    const void* w;
    const void* bias;               /* NULL or [n] */
    int32_t m, n, k, silu_inter;
    int64_t x_row_stride, out_row_stride;
    const void* norm_weight;        /* NULL or [k] */
    float norm_eps;
    int32_t epilogue;
    const int64_t* positions;       /* ROPE_STORE only, below */
    const float* cos_sin;
    void* k_cache;
    void* v_cache;
    const int32_t* slot_mapping;
    int32_t h, kvh, hd;
    int32_t norm_folded;
    /* streaming form (csrc/linear_stream.hip), all optional: */
    int32_t x_packed;               /* x is in MFMA-fragment order [ceil(m/16)][k/32][64][8] (nvh_pack_index); x_row_stride unused */
    void* out_packed;               /* NULL or: the epilogue also writes its bf16 result in fragment order
                                       ([ceil(m/16)][cols/32][64][8], cols = n, or silu_inter for SILU_MUL); `out` may then be
                                       NULL for NONE / SILU_MUL */
    void* workspace;                /* NULL or nvh_linear_small_m_workspace() bytes, ZERO-FILLED once by the caller (the
                                       kernel leaves its tickets zero); needed when k > 1024: K is then split over
                                       workgroups and the last-arriving one sums the partials in a fixed order */
    size_t workspace_bytes;
    /* greedy candidates (NONE epilogue, k <= 1024): every workgroup also writes, per row, the largest bf16 output among its
       columns and that column's index to candidate_val / candidate_idx [workgroup * candidate_stride + row]
       (nvh_linear_small_m_candidate_groups() workgroups; ties -> lowest column).  With candidates `out` may be NULL: the LM
       head + arg-max of a greedy decode step then never materialises the logits (layers/embed_head.py:66 +
       layers/sampler.py at temperature 0); finish with nvh_greedy_advance_candidates. */
    float* candidate_val;
    int32_t* candidate_idx;
    int64_t candidate_stride;
    /* prefetch hint (streaming form, optional): device memory the NEXT launches on this stream will stream once — typically the
       weights of the following projection.  A decode-sized projection occupies 36-224 of the device's CUs; the workgroups this
       launch adds for the idle ones read the range (default cache policy) and drop it, so that the later launch finds its operand
       in the caches.  Pure hint: results do not depend on it, only whole lines inside [prefetch, prefetch + prefetch_bytes) are
       read, NULL / 0 = none; ranges above 4 MiB are ignored (large prefetches cost the launch more than they save). */
    const void* prefetch;
    size_t prefetch_bytes;
    /* SILU_MUL with glu_alpha != 0: the clamped gated unit of nvh_clamped_glu (limit glu_limit) instead of SiLU(g) * u */
    float glu_limit, glu_alpha;
    /* SILU_MUL with glu_gelu != 0: gelu_tanh(g) * u (nvh_gelu_glu) instead */
    int32_t glu_gelu;
    /* NONE with x_packed, x_groups > 1: weight rows come in groups of x_group_rows (a multiple of 16; the last group may have any multiple of 16), group g is
       applied to the activations at x + g * x_group_stride elements */
    int32_t x_groups, x_group_rows, x_group_stride;
} nvh_linear_desc;
int nvh_linear_small_m_ex(const nvh_linear_desc* desc, int dtype, void* stream);
/* residual[n_rows, hidden] += y (bf16, one rounding — the add of add_rms_forward, layers/layernorm.py:35-36) and, if `packed` is
 * not NULL, the updated rows again in fragment order for the next nvh_linear_small_m_ex with x_packed: the step between a
 * tensor-parallel all-reduce of a row-parallel projection (layers/linear.py:185-190) and the next projection. */
int nvh_residual_add_pack(void* residual, const void* y, void* packed, int n_rows, int hidden, int64_t residual_row_stride,
                          int64_t y_row_stride, int dtype, void* stream);
size_t nvh_linear_small_m_workspace(int m, int n, int k, int epilogue);
int nvh_linear_small_m_candidate_groups(int n, int k);      /* candidate records per row of a NONE launch; 0 = unsupported shape */

/*
 * "Next" row (taken to its end): the front of a decode layer as ONE call — the fused qkv projection
 * (+ folded RMSNorm, bias, RoPE, K/V store) and the decode attention on its output.  Replaces the sequence nanovllm/models/qwen3.py:104-117
 * (qkv_proj -> rotary_emb -> self.attn) with nanovllm/layers/attention.py:84-86 (store_kvcache) and :99-101 (flash_attn_with_kvcache)
 * inside it.  Result: that of nvh_linear_small_m_ex(qkv) followed by nvh_paged_decode_packed on the q rows it wrote.
 *   qkv            a NVH_EPI_ROPE_STORE descriptor (see nvh_linear_small_m_ex): out = the q rows [m, h*hd], k_cache / v_cache /
 *                  slot_mapping = where this step's K / V rows go; prefetch = the output projection's weights (optional hint)
 *   attn_out       [m, h, hd] bf16; attn_out_packed: NULL or the same rows in fragment order (as nvh_paged_decode_packed)
 *   block_tables / context_lens / block_size / max_blocks / bt_row_stride / scale   as nvh_paged_decode (context_lens COUNT the token
 *                  this step stores, model_runner.py:252-258; rows with context 0 give zeros)
 *   workspace      nvh_paged_decode_workspace(m, h, hd, max_blocks, block_size) bytes, zero-filled once
 * Three forms were built and measured on MI355X (profiles/r03_qkv_attend_*); nvh_qkv_rope_attend runs the winner,
 * nvh_qkv_rope_attend_variant reaches all of them (tests and A/B):
 *   mode 1  TWO launches (the projection, then the attention call).  The winner at every shape tried; mode 0 = this.
 *   mode 2  ONE launch (csrc/qkv_attend.hip): producer workgroups compute the projection's tiles and publish q and the new K/V rows
 *           write-through; the attention workgroups start their K/V stream with the launch and wait (bounded) only for those.  Needs
 *           hd == 64, k <= 1024 (no split-K), x_packed, norm_folded, h / kvh <= 16, kvh <= 15 and a grid of at most two workgroups
 *           per CU (all resident: consumers wait for producers) on a device this stream has to itself; NVH_E_SHAPE otherwise.
 *           q and the cache rows are the same bits as mode 1's, the attention output the same bits as NVH_DECODE_CHUNKED_P128's.
 *           2.2 us per layer SLOWER than mode 1 at Qwen2-0.5B bs = 32: the stream's 16+ MB in flight queue in front of every load of the
 *           producer -> consumer chain.  A consumer whose wait runs out (~1 s) writes NaN rows and sets a status word instead of
 *           hanging (nvh_qkv_rope_attend_status, host-synchronous); spin_limit > 0 shortens the wait; missing_producers > 0 makes
 *           every consumer wait for producers that do not exist (the time-out path).
 *   mode 3  mode 1 with the projection launch's idle CUs touching the first `spin_limit` (default 1) passes of every attention workgroup's
 *           K/V into the caches (hd 64).  +1.3 % on the decode step with one pass, +5 % with two: a loss as well.
 * *one_launch (nullable) reports whether the one-launch kernel ran.  Capture-safe in every mode.
 */
int nvh_qkv_rope_attend(const nvh_linear_desc* qkv, void* attn_out, void* attn_out_packed,
                        const int32_t* block_tables, const int32_t* context_lens, int block_size, int max_blocks,
                        int64_t bt_row_stride, float scale, int dtype, void* workspace, size_t workspace_bytes, void* stream);
int nvh_qkv_rope_attend_variant(int mode, uint32_t spin_limit, int missing_producers, int* one_launch,
                                const nvh_linear_desc* qkv, void* attn_out, void* attn_out_packed,
                                const int32_t* block_tables, const int32_t* context_lens, int block_size, int max_blocks,
                                int64_t bt_row_stride, float scale, int dtype, void* workspace, size_t workspace_bytes, void* stream);
int nvh_qkv_rope_attend_status(const void* workspace, uint32_t* timed_out);
/* nvh_greedy_advance on candidate records instead of logits: token = column of the best candidate of each row */
int nvh_greedy_advance_candidates(const float* candidate_val, const int32_t* candidate_idx, int groups, int64_t candidate_stride,
                                  int n_rows, int64_t* input_ids, int64_t* positions, int32_t* context_lens, int32_t* slot_mapping,
                                  const int32_t* block_tables, int64_t bt_row_stride, int block_size,
                                  int64_t* tokens_log, int64_t log_row_stride, int64_t* row_steps, void* stream);
/* The same, and the NEXT step's token embedding in the same launch (VocabParallelEmbedding.forward at tp = 1,
 * nanovllm/layers/embed_head.py:34-45): hidden_out[r, :] = embed_weight[input_ids[r], :] with the token just chosen (rows with
 * context_lens 0 keep their token), and, if hidden_packed is not NULL, the same rows in fragment order for a following
 * nvh_linear_small_m_ex with x_packed.  embed_weight [vocab, hidden] bf16 contiguous, hidden % 32 == 0, 16-byte aligned buffers.
 * The chosen token is always a valid row of embed_weight: arg-max follows torch.argmax (NaN counts as the maximum, ties -> lowest
 * index, an all -inf row -> 0) and the index is clamped to [0, vocab). */
int nvh_greedy_advance_candidates_embed(const float* candidate_val, const int32_t* candidate_idx, int groups, int64_t candidate_stride,
                                        int n_rows, int64_t* input_ids, int64_t* positions, int32_t* context_lens, int32_t* slot_mapping,
                                        const int32_t* block_tables, int64_t bt_row_stride, int block_size,
                                        int64_t* tokens_log, int64_t log_row_stride, int64_t* row_steps,
                                        const void* embed_weight, int vocab, int hidden, void* hidden_out, int64_t hidden_row_stride, void* hidden_packed,
                                        int dtype, void* stream);
/* offset (in elements) of activation element (row, col) of an [m, cols] matrix in fragment order */
int64_t nvh_pack_index(int row, int col, int cols);

/*
 * "Next" row: the step immediately AFTER attention under tensor parallelism — the all-reduce of the
 * row-parallel projections' partial sums (RowParallelLinear.forward, nanovllm/layers/linear.py:185-190: dist.all_reduce over
 * NCCL) with the residual add that follows it (add_rms_forward, nanovllm/layers/layernorm.py:35-36) fused in.  One-shot over
 * xGMI instead of RCCL's ring: every rank maps every peer's staging buffer and flag table through hipIpc handles, signals with
 * one remote store per peer, reads the p-1 peers' partials over p-1 distinct links at once and sums in rank order in fp32 (all
 * ranks produce the same bits).  Decode-sized messages ([<= 64, hidden] bf16); capture-safe; no trailing barrier (staging is
 * double-buffered by a device-resident epoch).  A dead peer ends in NaN rows and a failure mark, not a hang.
 *
 * Set-up (host-synchronous, once, NOT capturable), per rank:
 *   nvh_comm_alloc(&stage, nvh_allreduce_stage_bytes(max_rows, hidden));   nvh_comm_alloc(&flags, nvh_allreduce_flag_bytes(world));
 *   nvh_comm_alloc(&state, 64);                                            (zero-filled fine-grained device memory)
 *   nvh_comm_ipc_export(stage / flags, handle[NVH_COMM_IPC_HANDLE_BYTES]) -> exchange the handles by any host channel ->
 *   nvh_comm_ipc_open(peer handle, &peer_ptr) for every peer; upload the two [world] pointer tables (own pointers at [rank])
 *   to device memory.  `state` stays local.
 * Call (every rank, same order of calls, same rows / hidden):
 *   x              [rows, hidden] bf16 partial sums of this rank (row stride x_row_stride elements)
 *   epilogue       NVH_AR_EPI_NONE: out[rows, hidden] = bf16(sum over ranks);  out may alias x
 *                  NVH_AR_EPI_RESIDUAL_ADD: out is the residual stream: out = bf16(out + bf16(sum)); packed (nullable): the
 *                  updated rows again in fragment order (nvh_pack_index) for the next nvh_linear_small_m_ex with x_packed
 *   stage_bytes    size of EACH rank's staging buffer (>= nvh_allreduce_stage_bytes(rows, hidden))
 *   state          uint32[16], local: [0] calls completed, [2] != 0 after a peer timed out OR was found two calls ahead (the epoch that
 *                  failed; that call's rows are NaN), [3] if non-zero replaces the poll limit (tests force the time-out with it)
 * nvh_allreduce_status (host-synchronous: waits for the device, NOT capturable) reads those two words back.
 */
#define NVH_COMM_IPC_HANDLE_BYTES 64
enum { NVH_AR_EPI_NONE = 0, NVH_AR_EPI_RESIDUAL_ADD = 1 };
int nvh_comm_alloc(void** ptr, size_t bytes);
int nvh_comm_free(void* ptr);
int nvh_comm_ipc_export(void* ptr, void* handle_out);
int nvh_comm_ipc_open(const void* handle, void** ptr);
int nvh_comm_ipc_close(void* ptr);
size_t nvh_allreduce_stage_bytes(int max_rows, int hidden);
size_t nvh_allreduce_flag_bytes(int world);
int nvh_allreduce_status(const void* state, uint32_t* calls_completed, uint32_t* failed_epoch);
int nvh_allreduce_oneshot(void* out, const void* x, void* packed, void* const* stage_ptrs, void* const* flag_ptrs, void* state,
                          int world, int rank, int rows, int hidden, int64_t x_row_stride, int64_t out_row_stride,
                          size_t stage_bytes, int epilogue, int dtype, void* stream);

/* ================================================================================================================================
 * Layers with their own state: gated linear recurrence and latent attention, and the row ops of models that keep the residual stream in
 * fp32 and normalise a sublayer's output.  `dtype` is the activation type: NVH_BF16, or NVH_F32 for a true 32-bit model (every activation,
 * cache row and matrix operand is then float).  Widths ("cols") may be padded with zeros; the counts a mean runs over are given apart.
 */
/* x[rows, cols] (fp32) = embed[token] * scale; xb (nullable): the same in the activation type; packed
 * (nullable, bf16, cols % 32 == 0): in fragment order.  Tokens outside [0, vocab) are clamped.  table (nullable, fp32 [max_position, cols]): row
 * positions[row] of it is added; copy (nullable): the fp32 rows a second time. */
int nvh_embed_rows(float* x, void* xb, void* packed, const int64_t* tokens, const void* embed, float scale, int rows, int cols, int vocab, float* copy,
                   const int64_t* positions, const float* table, int max_position, int dtype, void* stream);
/* x += rmsnorm(y) * w (y given), or the result = rmsnorm(x) * w with x unchanged (y NULL). */
typedef struct nvh_norm_residual_desc {
    float* x;                    /* [rows, cols] fp32 residual stream */
    void* xb;                    /* nullable: the result in the activation type */
    void* packed;                /* nullable (bf16): the same rows in MFMA-fragment order */
    const void* y;               /* sublayer output [rows, cols] (residual form) or null: norm of x itself, x unchanged */
    const float* w;              /* [cols] multiplicative weight (a zero-centred weight has its one already added) */
    float eps;
    int32_t rows, cols, n;           /* n: elements the mean runs over (columns n.. are zero padding) */
    int64_t y_stride;
} nvh_norm_residual_desc;
int nvh_norm_residual(const nvh_norm_residual_desc* d, int dtype, void* stream);
/* out[rows, inter] = g sigmoid(alpha g) (u + 1), g = min(gate, limit), u = clamp(up, -limit, limit); gate_up rows hold gate | up. */
int nvh_clamped_glu(void* out, const void* gate_up, int rows, int inter, int64_t gate_up_row_stride, int64_t out_row_stride, float limit, float alpha,
                    int dtype, void* stream);
/* gelu(gate) * up, the tanh form of gelu. */
int nvh_gelu_glu(void* out, const void* gate_up, int rows, int inter, int64_t gate_up_row_stride, int64_t out_row_stride, int dtype, void* stream);
/* Real-gated linear recurrent unit behind a causal depthwise convolution: log a = -rate sigmoid(ra u), S = a S + sqrt(1 - a^2) sigmoid(ri u) u,
 * out = S gelu(y).  nvh_rglru_chunks: portions of prompts (and single tokens), cut by the caller into segments that are
 * scanned side by side; segments of one portion are consecutive.  nvh_rglru_step: row i is one new token of sequence i (bf16; nvh_rglru_step_supported(block)).
 * generic: 0 = the fastest form the shape allows, 1 = the plain kernel, 2 = the MFMA walk without LDS-DMA (tests). */
typedef struct nvh_rglru_desc {
    const void* yx;              /* [rows, 2 * width]: gate branch | recurrent branch (biases added), row stride yx_stride */
    int64_t yx_stride;
    int32_t width, block, blocks;    /* width == blocks * block, a multiple of 64; block % 32 == 0 */
    int32_t taps;
    const float* conv_w;         /* [taps, width], last row = the current token */
    const float* conv_b;         /* [width] */
    const void* ra;              /* [blocks, block, block] ([out, in]) */
    const void* ri;
    const float* ra_b;           /* [width] */
    const float* ri_b;
    const float* rate;           /* [width]: log a = -rate * r */
    const int32_t* chunks;       /* [n_chunks, 4]: first row, rows, sequence, index of the segment in its sequence's portion */
    int32_t n_chunks;
    int32_t segment;             /* tokens of every segment but a portion's last; a multiple of nvh_rglru_chunk_tokens() */
    int32_t summaries;           /* != 0: some portion has more than one segment */
    const int64_t* positions;    /* [rows] */
    const int32_t* state_slots;  /* [sequences]; < 0: nothing is read or kept */
    float* state;                /* [slots, width] */
    void* conv_state;            /* [slots, taps, width]: input of position p at ring entry p % taps */
    float* s_loc;                /* [n_chunks, width] scratch: value at a segment's end */
    float* a_cum;                /* [n_chunks, width] scratch: product of a segment's decays */
    void* out;                   /* [rows, width]: S * gelu(y), row stride out_stride */
    int64_t out_stride;
    void* out_packed;            /* nullable (bf16, step form): the result in MFMA-fragment order */
} nvh_rglru_desc;
int nvh_rglru_chunk_tokens(void);
int nvh_rglru_chunks(const nvh_rglru_desc* d, int generic, int dtype, void* stream);
int nvh_rglru_step(const nvh_rglru_desc* d, int rows, int dtype, void* stream);
int nvh_rglru_step_supported(int block);
/* Latent attention, row ops in front: query-latent norm, key-latent norm, rotation of interleaved pairs of the shared key part, cache store. */
typedef struct nvh_latent_prep_desc {
    const void* a;               /* [rows, a_stride]: query latent (q_cols) | key latent (kv_cols) | shared key part (rot_cols) */
    int64_t a_stride;
    int32_t rows, q_rank, q_cols, kv_rank, kv_cols, rot, rot_cols;   /* *_cols: padded widths; kv_cols == 0: no key latent in `a` */
    const float* q_w;            /* [q_cols] */
    const float* kv_w;           /* [kv_cols] */
    float eps;
    void* cq;                    /* [rows, q_cols] normed query latent */
    void* cq_packed;             /* nullable (bf16): in MFMA-fragment order instead */
    void* cache;                 /* [slots, kv_cols + rot_cols] */
    const int32_t* slots;        /* [rows]; < 0: not stored */
    const int64_t* positions;    /* [rows] */
    const float* cos_sin;        /* [max_position, rot]: cos(0..rot/2) | sin(0..rot/2) */
    int32_t max_position;
} nvh_latent_prep_desc;
int nvh_latent_prep(const nvh_latent_prep_desc* d, int dtype, void* stream);
/* Latent attention in the cache's own space: queries absorbed through w_uk, attention over the shared rows, values through w_uv.  Three launches;
 * generic != 0 forces the plain attention kernel (tests).  bf16 and nvh_latent_attend_mfma(kv_cols, rot_cols, block_size) and row_seq == NULL:
 * MFMA tiles; anything else: the plain kernel (kv_cols <= 2048). */
typedef struct nvh_latent_attn_desc {
    /* queries */
    const void* q;               /* [rows, heads, dim_cols + qrot_cols] (row stride q_stride): unrotated | rotated part, not rotated yet */
    int64_t q_stride;
    int32_t rows, heads, dim_cols, qrot_cols;
    /* cache */
    const void* cache;           /* pages of block_size rows [kv_cols + rot_cols] */
    int32_t kv_cols, rot, rot_cols, block_size;
    const int32_t* block_tables; /* [sequences, bt_stride] */
    int64_t bt_stride;
    int32_t max_blocks;
    const int32_t* row_seq;      /* nullable: sequence of a row (null: row i is sequence i) */
    const int64_t* positions;    /* [rows]; a row sees positions 0 .. its own */
    const float* cos_sin;
    int32_t max_position;
    const void* w_uk;            /* [heads, kv_cols, dim_cols] */
    const void* w_uv;            /* [heads, v_cols, kv_cols] */
    int32_t v_cols;
    float scale;
    /* scratch and result */
    void* qa;                    /* [rows, heads, kv_cols + rot_cols]: queries in the latent space */
    float* part_o;               /* [rows, splits, heads, kv_cols] un-normalised */
    float* part_ml;              /* [rows, splits, heads, 2]: running max (log2 domain), sum */
    int32_t splits;
    void* out;                   /* [rows, heads * v_cols], row stride out_stride */
    int64_t out_stride;
    void* out_packed;            /* nullable (bf16) */
} nvh_latent_attn_desc;
int nvh_latent_attention(const nvh_latent_attn_desc* d, int generic, int dtype, void* stream);
int nvh_latent_attend_mfma(int kv_cols, int rot_cols, int block_size);
/* out[total, cols] = the cache rows of every key of the sequences, in order (cu_k: [batch + 1] key offsets). */
int nvh_latent_gather(void* out, const void* cache, const int32_t* cu_k, const int32_t* block_tables, int64_t bt_stride, int batch, int total, int cols,
                      int block_size, int dtype, void* stream);
/* Causal attention of prompt portions over expanded keys and values (bf16, bottom-right aligned mask), key width dk != value width dv. */
typedef struct nvh_latent_prefill_desc {
    const uint16_t* q;           /* [rows, heads, dk] unrotated | rotated part (not rotated yet), row stride q_stride */
    const uint16_t* k;           /* [keys, heads, dim_cols], row stride k_stride */
    const uint16_t* k_rot;       /* [keys, dk - dim_cols] shared rotated part, row stride kr_stride */
    const uint16_t* v;           /* [keys, heads, dv], row stride v_stride */
    uint16_t* out;               /* [rows, heads * dv], row stride out_stride */
    int64_t q_stride, k_stride, kr_stride, v_stride, out_stride;
    const int32_t* cu_q;         /* [batch + 1] */
    const int32_t* cu_k;
    const int64_t* positions;    /* [rows] */
    const float* cos_sin;
    int32_t max_position, rot;
    int32_t batch, heads, dim_cols, dk, dv, max_q;
    float scale_log2;
} nvh_latent_prefill_desc;
int nvh_latent_prefill(const nvh_latent_prefill_desc* d, int dtype, void* stream);
int nvh_latent_prefill_supported(int dk, int dv);

/* ================================================================================================================================
 * Softmax attention over pages with windows, kept first tokens and sinks; lightning attention; mixture of experts; row ops of models whose
 * sublayers share one layer norm.  `dtype` and "cols" as in the section above.
 *
 * Cache pages of one attention layer: [pages][kv_heads][block_size rows of dk keys, then block_size rows of dv values].
 */
/* Row ops behind a q | k | v projection, in place: optional RMS norm over all query columns and over all key columns at once, rotation of
 * interleaved pairs of queries and keys, keys and values into the cache. */
typedef struct nvh_attn_prep_desc {
    void* qkv;                   /* [rows, heads * dk | kv_heads * dk | kv_heads * dv], row stride qkv_stride; queries are rewritten */
    int64_t qkv_stride;
    int32_t rows, heads, kv_heads, dk, dv;
    const float* q_w;            /* nullable: [heads * dk] norm weight (then k_w too) */
    const float* k_w;            /* [kv_heads * dk] */
    int32_t q_n, k_n;            /* columns the means run over (the rest is zero padding) */
    float eps;
    const int64_t* positions;    /* [rows] */
    const float* cos_sin;        /* [max_position, rot]: cos(0..rot/2) | sin(0..rot/2) */
    int32_t max_position, rot;   /* rot <= dk: leading dimensions of a head that turn */
    void* cache;
    const int32_t* slots;        /* [rows] page * block_size + offset; < 0: not stored */
    int32_t block_size;
    int32_t head_norm;           /* != 0: the norms run over every head by itself; q_w and k_w are [dk], shared by the heads, q_n and k_n the columns of a head */
    const float* v_cos_sin;      /* nullable: values turn too, [max_position, v_rot] as cos_sin, the first v_rot <= dv dimensions of every head */
    int32_t v_rot;
} nvh_attn_prep_desc;
int nvh_attn_prep(const nvh_attn_prep_desc* d, int dtype, void* stream);
/* softmax(scale q . k) v over the keys a query sees: position j of its sequence if j <= its own and (window == 0 or nearer than `window` or
 * j < keep_first); with chunk > 0 (window 0) instead of a window: j / chunk == its own / chunk, or j < keep_first.  o_cos_sin (nullable): a head's output at
 * position p is turned back, interleaved pairs of its first o_rot dimensions by minus the angles of row p (values stored turned, see nvh_attn_prep).  sink (nullable): exp(sink[head]) joins the denominator.  Query head h reads key/value head h / (heads / kv_heads).
 *   rows form   (nvh_paged_attend_rows): row i belongs to sequence row_seq[i] (or i); splits > 1: context splits, merged by the last workgroup to arrive
 *   portions    (nvh_paged_attend_prompt, bf16): rows cu_q[b] .. of sequence b are its last ones, cu_k[b + 1] - cu_k[b] keys in all
 * MFMA / streaming forms for the widths nvh_paged_attend_supported names; `generic` (rows form): the plain kernel, any width up to 2048. */
typedef struct nvh_paged_attend_desc {
    const void* q;               /* [rows, heads, dk], row stride q_stride */
    int64_t q_stride;
    int32_t rows, heads, kv_heads, dk, dv;
    const void* cache;
    int32_t block_size;
    const int32_t* block_tables; /* [sequences, bt_stride] */
    int64_t bt_stride;
    const int32_t* row_seq;      /* nullable */
    const int64_t* positions;    /* [rows] (rows form) */
    const int32_t* cu_q;         /* [batch + 1] (portions) */
    const int32_t* cu_k;
    int32_t batch, max_q;
    float scale;
    int32_t window, keep_first;
    const float* sink;           /* nullable: [heads] */
    int32_t splits;
    float* part;                 /* splits > 1: [rows, heads, splits, dv + 4] scratch */
    uint32_t* tickets;           /* zero before the launch, left zero: nvh_paged_attend_ticket_bytes(rows, kv_heads, heads) */
    void* out;                   /* nullable: [rows, heads * dv], row stride out_stride */
    int64_t out_stride;
    void* out_packed;            /* nullable (bf16, rows form): the same in MFMA-fragment order */
    const float* talk;           /* nvh_talk_*: [heads, heads]; NULL otherwise */
    float softcap;               /* nvh_talk_*: 0 or the cap */
    float* scores;               /* nvh_talk_rows: [rows, span, nvh_talk_score_cols(heads)] scratch */
    int32_t span;                /* 64 times the most 64-key tiles a row sees */
    int32_t chunk;               /* not for nvh_talk_* */
    const float* o_cos_sin;      /* nullable: [max_position, o_rot]; not for nvh_talk_* */
    int32_t max_position, o_rot;
} nvh_paged_attend_desc;
int nvh_paged_attend_supported(int dk, int dv, int block_size);
size_t nvh_paged_attend_ticket_bytes(int rows, int kv_heads, int heads);
int nvh_paged_attend_rows(const nvh_paged_attend_desc* d, int generic, int dtype, void* stream);
int nvh_paged_attend_prompt(const nvh_paged_attend_desc* d, int dtype, void* stream);

/* The same attention with scores capped, softcap tanh(scale q . k / softcap), and then mixed across the heads, score_h <- sum_g talk[h][g] score_g, before the
 * softmax.  nvh_talk_rows is two launches (scores to memory, then the rest); nvh_talk_prompt is one, all heads of 16 rows in a workgroup: it takes caps in
 * (0, 1e4] and mixing matrices with entries of at most 2000 (both pass through pairs of fp16 numbers). */
int nvh_talk_rows_supported(int heads, int dk, int dv, int block_size);
int nvh_talk_score_cols(int heads);
size_t nvh_talk_ticket_bytes(int rows, int kv_heads, int heads);
int nvh_talk_rows(const nvh_paged_attend_desc* d, int generic, int dtype, void* stream);
int nvh_talk_prompt_supported(int heads, int kv_heads, int dk, int dv, int block_size, float softcap);
int nvh_talk_prompt(const nvh_paged_attend_desc* d, int dtype, void* stream);

/* Lightning attention: per head S = decay S + k v^T, o = S^T q with q, k, v = silu of the projection's columns (rounded to the activation type);
 * the state is fp32.  nvh_lightning_chunks: portions cut into segments as for nvh_rglru_chunks; nvh_lightning_step: row i is one new token of
 * sequence i.  A token at position 0 takes the state as zero.  generic (chunks): the plain token-by-token kernel, any width; the MFMA form and the step need
 * nvh_lightning_supported(dk, dv). */
typedef struct nvh_lightning_desc {
    const void* qkv;             /* [rows, heads * dk | heads * dk | heads * dv], row stride qkv_stride */
    int64_t qkv_stride;
    int32_t rows, heads, dk, dv;
    const float* decay;          /* [heads] */
    const int64_t* positions;    /* [rows] */
    const int32_t* state_slots;  /* [sequences]; < 0: nothing is read or kept */
    float* state;                /* [slots, heads, dk, dv] */
    const int32_t* chunks;       /* [n_chunks, 4]: first row, rows, sequence, index of the segment in its sequence's portion */
    int32_t n_chunks;
    int32_t summaries;           /* != 0: some portion has more than one segment */
    float* seg_state;            /* summaries: [n_chunks, heads, dk, dv] scratch */
    void* out;                   /* [rows, heads * dv], row stride out_stride */
    int64_t out_stride;
} nvh_lightning_desc;
int nvh_lightning_supported(int dk, int dv);
int nvh_lightning_chunks(const nvh_lightning_desc* d, int generic, int dtype, void* stream);
int nvh_lightning_step(const nvh_lightning_desc* d, int dtype, void* stream);
/* out = rmsnorm(x over n columns) * w * sigmoid(gate); packed (nullable, bf16): in fragment order instead. */
int nvh_norm_gate(void* out, void* packed, const void* x, const void* gate, const float* w, float eps, int rows, int cols, int n, int64_t x_stride,
                  int64_t gate_stride, int64_t out_stride, int dtype, void* stream);

/* Mixture of experts.  Route: s = sigmoid(h . router_e) in 32-bit; choice scores s + correction; the experts form `groups` equal groups of neighbours,
 * a group counts the sum of its two largest choice scores, the best `keep` groups stay open, the `top` largest choice scores among them win;
 * weights s / (sum + 1e-20) * scale.  softmax != 0: the scores are the logits themselves, `correction` a bias on them (choice and weights), groups 1, the weights
 * the softmax over the chosen scores, times scale.  Pair p = row * top + k. */
typedef struct nvh_moe_route_desc {
    const void* x;               /* [rows, cols], row stride x_stride */
    int64_t x_stride;
    const void* router;          /* [experts, cols] */
    const float* correction;     /* [experts] */
    int32_t rows, cols, experts, top, groups, keep;
    float scale;
    int32_t* ids;                /* [rows, top] */
    float* weights;              /* [rows, top] */
    int32_t softmax;
} nvh_moe_route_desc;
int nvh_moe_route(const nvh_moe_route_desc* d, int dtype, void* stream);
/* Pairs sorted by expert: slot_pair[slot], tiles [max_tiles][4] = (expert, first slot, slots, tiles in use), unused ones with
 * 0 slots, tile_rows slots each;
 * counts: [nvh_moe_dispatch_blocks(pairs), experts] scratch.  max_tiles >= pairs / tile_rows + experts. */
int nvh_moe_dispatch_blocks(int pairs);
int nvh_moe_dispatch(int32_t* slot_pair, int32_t* tiles, int32_t* counts, const int32_t* ids, int pairs, int experts, int tile_rows, int max_tiles, void* stream);
/* Expert products.  glu: act[p] = silu(x[p / top] . gate_e) * (x . up_e), w = [experts, 2 * n, k] (gate rows, then up rows), or with alpha != 0 the clamped unit
 * g sigmoid(alpha g) (u + 1), g = min(gate, limit), u = clamp(up, -limit, limit); otherwise
 * out[p] = x[p] . w_e, w = [experts, n, k].
 * tiles == NULL: small batches (bf16, at most 64 rows), the pairs of an expert found from ids; otherwise tiles of tile_rows from
 * nvh_moe_dispatch (bf16: 128 or 256, f32: 64; nvh_moe_tile_rows picks).  n and k multiples of 64. */
typedef struct nvh_moe_gemm_desc {
    void* out;                   /* [pairs, n] */
    const void* x;               /* glu: [rows, k], row stride x_stride; otherwise [pairs, k] */
    int64_t x_stride;
    const void* w;
    int32_t pairs, top, experts, n, k, glu;
    const int32_t* ids;          /* [pairs] (small form) */
    const int32_t* slot_pair;    /* [pairs] */
    const int32_t* tiles;
    int32_t max_tiles, tile_rows;
    float limit, alpha;
} nvh_moe_gemm_desc;
int nvh_moe_tile_rows(int pairs, int experts, int dtype);
int nvh_moe_gemm(const nvh_moe_gemm_desc* d, int dtype, void* stream);

/* x (fp32 stream) += mult * P(y + sum_k ew[row, k] * e[row * top + k])  (each part nullable; P: the layer norm with post_w and post_b where given, nothing
 * otherwise), x += base, x += shift, then, with w given, the layer norm of the new row: (x - mean) / sqrt(var + eps) * w + b. */
typedef struct nvh_residual_norm_desc {
    float* x;                    /* [rows, cols] */
    const void* y;               /* nullable: [rows, cols], row stride y_stride */
    int64_t y_stride;
    const void* e;               /* nullable: [rows * top, cols] expert outputs */
    const float* ew;             /* [rows, top] */
    int32_t top;
    const float* w;              /* nullable: no norm */
    const float* b;
    float eps;
    int32_t rows, cols, n;       /* n: elements mean and variance run over */
    void* xb;                    /* nullable: the normed rows in the activation type */
    void* packed;                /* nullable (bf16): the same in MFMA-fragment order */
    const float* post_w;         /* nullable: [cols] */
    const float* post_b;
    float mult;
    const float* base;           /* nullable: [rows, cols] */
    const float* shift;          /* nullable: [cols] */
} nvh_residual_norm_desc;
int nvh_residual_norm(const nvh_residual_norm_desc* d, int dtype, void* stream);
/* out = coef[0] N(z) + coef[1] N(z^2) + coef[2] N(z^3) + coef[3], powers by element, N(v) = v / sqrt(mean over n columns of v^2 + eps); zero past n. */
int nvh_poly_norm(void* out, void* packed, const void* z, const float* coef, float eps, int rows, int cols, int n, int64_t z_stride, int64_t out_stride, int dtype, void* stream);
/* x = cap * tanh(x / cap) in place, rows of `cols` elements. */
int nvh_softcap(void* x, float cap, int rows, int cols, int64_t stride, int dtype, void* stream);

/* ---- several residual streams, and what looks at the token before (csrc/streams.hip).
 * Portions: row_seq [rows] and cu_rows [sequences + 1] give every row's sequence and the rows of a sequence's portion; both NULL: row i is the one new token of
 * sequence i.  Rings hold a sequence's last rows, [slots, depth, cols] in the activation type, the row of position p at entry p % depth.  state_slots < 0: nothing
 * is read or kept; nothing is read before position 0. */
/* x = embed[token] + bigram[b], b = (previous token * mul_prev + token * mul_cur) mod buckets, or row `buckets` for a sequence's first token. */
typedef struct nvh_bigram_embed_desc {
    float* x;                    /* [rows, cols] */
    const int64_t* tokens;       /* [rows] */
    const int64_t* positions;    /* [rows] */
    const int32_t* row_seq;
    const int32_t* cu_rows;
    const int32_t* state_slots;  /* [sequences] */
    int64_t* last_token;         /* [slots] */
    const void* embed;           /* [vocab, cols] */
    const void* bigram;          /* [buckets + 1, cols] */
    int64_t buckets, mul_prev, mul_cur;
    int32_t rows, cols, vocab;
} nvh_bigram_embed_desc;
int nvh_bigram_embed(const nvh_bigram_embed_desc* d, int dtype, void* stream);

/* Hyper-connections: with y given, x_t <- sum_s mix[s][t] x_s + out[t] y for all streams at once (to xout, if given); y2 given: y is first replaced by
 * y_scale (rms(y) y_w + rms(y2) y2_w), means over n columns.  u = sum_s in[s] x_s (in NULL: plain sum) of the new streams goes to `sum`, and, with w given, its RMS
 * norm in `groups` equal parts of the n columns, times w, to h and / or `packed`.  shift given (bf16, row i is one new token of sequence i): nvh_token_shift of the
 * normed rows in the same launch, in fragment order to `shifted`. */
typedef struct nvh_stream_mix_desc {
    const float* xin;            /* stream s of row r at xin + r * xin_row + s * xin_stream (xin_stream 0: all streams alike) */
    int64_t xin_row, xin_stream;
    float* xout;                 /* nullable: [rows, streams, cols]; may be xin */
    int32_t rows, cols, n, streams;
    const void* y;               /* nullable: [rows, cols] */
    int64_t y_stride;
    const void* y2;              /* nullable */
    int64_t y2_stride;
    const float* y_w;
    const float* y2_w;
    float y_scale;
    const float* mix;            /* [streams, streams], [from][to] */
    const float* out;            /* [streams] */
    const float* in;             /* nullable: [streams] */
    float* sum;                  /* nullable: [rows, cols] */
    const float* w;              /* nullable: [cols], zero past n */
    int32_t groups;
    float eps;
    void* h;                     /* nullable: [rows, cols] in the activation type */
    void* packed;                /* nullable (bf16): the same in MFMA-fragment order */
    const float* shift;          /* nullable: [cols]; the following as in nvh_token_shift_desc */
    const float* mu;
    int32_t mixes, depth;
    void* ring;
    void* shifted;
    int64_t shifted_mix;
    const int64_t* positions;
    const int32_t* state_slots;
} nvh_stream_mix_desc;
int nvh_stream_mix(const nvh_stream_mix_desc* d, int dtype, void* stream);

/* s = h + (h' - h) shift with h' the previous token's h; mixes == 0: out = s; otherwise out[k] = s + (s' - s) mu[k] with s' the previous token's s (zeros before the
 * first token).  Depth of the ring: 2 without mixes, 3 with. */
typedef struct nvh_token_shift_desc {
    const void* h;               /* [rows, cols], row stride h_stride */
    int64_t h_stride;
    int32_t rows, cols;
    const float* shift;          /* [cols] */
    const float* mu;             /* [mixes, cols] */
    int32_t mixes;
    void* out;                   /* [max(mixes, 1)][rows, cols], out_mix elements apart; packed != 0 (bf16): each in MFMA-fragment order */
    int64_t out_mix;
    int32_t packed;
    void* ring;
    int32_t depth;
    const int64_t* positions;
    const int32_t* row_seq;
    const int32_t* cu_rows;
    const int32_t* state_slots;
    int32_t sequences;
} nvh_token_shift_desc;
int nvh_token_shift(const nvh_token_shift_desc* d, int dtype, void* stream);

/* silu(b + sum over taps of w[tap] x), the last tap on the current token; ring of `taps` rows. */
typedef struct nvh_causal_conv_desc {
    const void* x;               /* [rows, cols], row stride x_stride */
    int64_t x_stride;
    int32_t rows, cols, taps;
    const float* w;              /* [taps, cols] */
    const float* b;              /* [cols] */
    void* out;                   /* nullable: [rows, cols] */
    void* packed;                /* nullable (bf16): the same in MFMA-fragment order */
    void* ring;
    const int64_t* positions;
    const int32_t* row_seq;
    const int32_t* cu_rows;
    const int32_t* state_slots;
    int32_t sequences;
} nvh_causal_conv_desc;
int nvh_causal_conv(const nvh_causal_conv_desc* d, int dtype, void* stream);

/* Selective scan: S[c][n] <- exp(dt_c A[c][n]) S[c][n] + dt_c x_c B[n], y_c = sum_n S[c][n] C[n] + d_c x_c, out = y silu(z), dt = softplus(. + dt_bias).  The state is
 * fp32; a token at position 0 takes it as zero.  nvh_scan_states(n): the number of states kept for n of them (0: too many).
 *   portions (nvh_scan_chunks)  dt [rows, inner]; cut into segments as for nvh_rglru_chunks
 *   single   (nvh_scan_step)    bf16; row i is one new token of sequence i; dt [rows, rank] is multiplied by w_dt [inner, rank] first */
typedef struct nvh_scan_desc {
    const void* x;               /* [rows, inner] */
    int64_t x_stride;
    const void* dt;
    int64_t dt_stride;
    const float* dt_bias;        /* [inner] */
    const void* bc;              /* [rows, n | n]: B | C */
    int64_t bc_stride;
    const void* z;               /* [rows, inner] */
    int64_t z_stride;
    const float* a_log2;         /* [inner, n]: A log2(e) */
    const float* d;              /* [inner] */
    int32_t rows, inner, n;
    const int64_t* positions;    /* [rows] */
    const int32_t* state_slots;  /* [sequences]; < 0: nothing is read or kept */
    float* state;                /* [slots, inner, n] */
    const int32_t* chunks;       /* [n_chunks, 4]: first row, rows, sequence, index of the segment in its sequence's portion */
    int32_t n_chunks;
    int32_t summaries;           /* != 0: some portion has more than one segment */
    float* seg_state;            /* summaries: [n_chunks, inner, n] scratch */
    float* seg_dt;               /* summaries: [n_chunks, inner] scratch */
    const void* w_dt;
    int32_t rank;
    void* out;                   /* [rows, inner], row stride out_stride (single tokens: nullable) */
    int64_t out_stride;
    void* out_packed;            /* nullable (single tokens): the same in MFMA-fragment order */
} nvh_scan_desc;
int nvh_scan_states(int n);
int nvh_scan_chunks(const nvh_scan_desc* d, int dtype, void* stream);
int nvh_scan_step(const nvh_scan_desc* d, int dtype, void* stream);

/* Time mixing: per head o = (S + diag(u) k v^T)^T r, S <- diag(w) S + k v^T with w = exp(-exp(z + w0)) per token and key channel, then
 * out = o / sqrt(mean over n columns of o^2 + eps) * norm * silu(g).  The state is fp32; a token at position 0 takes it as zero.
 *   portions (nvh_wkv_chunks)  z [rows, heads * dim]; cut into segments as for nvh_rglru_chunks; generic: the plain token-by-token kernel, any width
 *   single   (nvh_wkv_step)    bf16; row i is one new token of sequence i; z [rows, rank]: w2 tanh(z) is computed first; nvh_wkv_supported(dim) */
typedef struct nvh_wkv_desc {
    const void* r;               /* r, k, v, g: [rows, heads * dim], one row stride */
    const void* k;
    const void* v;
    const void* g;
    int64_t stride;
    const void* z;
    int64_t z_stride;
    const float* w0;             /* [heads * dim] */
    const float* u;              /* [heads * dim] */
    const float* norm;           /* [heads * dim] */
    float eps;
    int32_t n;                   /* columns of a head that count (the rest is zero padding) */
    int32_t rows, heads, dim;
    const void* w2;              /* [heads * dim, rank] */
    int32_t rank;
    const int64_t* positions;    /* [rows] */
    const int32_t* state_slots;  /* [sequences]; < 0: nothing is read or kept */
    float* state;                /* [slots, heads, dim, dim]: [key][value] */
    const int32_t* chunks;       /* [n_chunks, 4]: first row, rows, sequence, index of the segment in its sequence's portion */
    int32_t n_chunks;
    int32_t summaries;           /* != 0: some portion has more than one segment */
    float* seg_state;            /* summaries: [n_chunks, heads, dim, dim] scratch */
    float* seg_decay;            /* summaries: [n_chunks, heads * dim] scratch */
    void* out;                   /* [rows, heads * dim], row stride out_stride (single tokens: nullable) */
    int64_t out_stride;
    void* out_packed;            /* nullable (single tokens): the same in MFMA-fragment order */
} nvh_wkv_desc;
int nvh_wkv_supported(int dim);
int nvh_wkv_chunks(const nvh_wkv_desc* d, int generic, int dtype, void* stream);
int nvh_wkv_step(const nvh_wkv_desc* d, int dtype, void* stream);

#ifdef __cplusplus
}
#endif
#endif /* NVH_ATTN_H */
