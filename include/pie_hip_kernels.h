/*
 * pie_hip_kernels.h — C ABI of the gfx950 (MI355X) kernel library behind the
 * Pie driver forward pass.
 *
 * Every entry point takes plain device pointers, shapes and a HIP stream
 * (passed as `void*`, i.e. a `hipStream_t`; NULL = the default stream), does no
 * allocation, keeps no global state, never throws, and returns a status code.
 * The functions replace, one for one, the `launch_*` C++ launchers of the
 * reference CUDA driver (the .hpp files under driver/cuda/src/kernels and driver/cuda/src/ops);
 * each declaration cites the launcher whose contract it follows.
 *
 * Conventions
 *   - bf16 tensors are raw 16-bit words (`uint16_t`), row-major.
 *   - "act x W" products follow the reference: act[M,K] · W[N,K]^T -> y[M,N]
 *     (driver/cuda/src/ops/gemm.hpp:152-160).
 *   - `beta` is 0 (overwrite y) or 1 (y += result, the residual fuse of
 *     driver/cuda/src/model/llama_like.cpp:626-628).
 */
#ifndef PIE_HIP_KERNELS_H
#define PIE_HIP_KERNELS_H

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

/* RoPE pairings of the rotation kernels and fused epilogues */
#define PIE_HIP_ROPE_HALF 0
#define PIE_HIP_ROPE_ADJACENT 1
#define PIE_HIP_ROPE_HALF_PAIRED_ROWS 2

#define PIE_HIP_OK 0
#define PIE_HIP_ERR_INVALID 1     /* null pointer, non-positive size, bad enum   */
#define PIE_HIP_ERR_UNSUPPORTED 2 /* shape the kernels do not cover              */
#define PIE_HIP_ERR_LAUNCH 3      /* HIP reported an error at launch             */

/* Library/ABI version: bumped on any change of a signature or of a memory layout an entry point
 * reads or writes.  A caller compares the macro it was built against with what the loaded
 * library returns and refuses to run on a mismatch (an old caller would link and compute
 * garbage).  History:
 *   1  first layout
 *   2  `pairing` argument of pie_hip_qkv_rope_fused / pie_hip_qkv_rope_skinny_tiled; `page_size`
 *      argument of pie_hip_kv_write_quant / pie_hip_qkv_rope_kvwrite_quant; KV scale pools
 *      [pages, hk, page_size] (were [pages, page_size, hk]); int4 tile-major weights in decode
 *      order (pie_hip_repack_mfma_tiles_int4); pie_hip_gemv_time_next removed
 *   3  lm_head argmax pairs, attention merge in the output projection, uniform-row hints
 *   4  the `swiglu` argument of the linears is an epilogue code (PIE_HIP_EPI_*: 0 and 1
 *      mean what they did, 2 is the squared ReLU); the layer-stack kernels
 *   5  epilogue code 3 (exact GELU); grouped attention with windows and sinks, memories with
 *      one decay per head, residual_norm
 *   6  gated products with biases and clamps (PieHipGlu, the *_glu entry points); gates on the
 *      outputs of grouped and latent attention; norms over whole projections; expert groups;
 *      residual_join
 *   7  current: `sinks` of latent attention, gates per head (`gate_cols`), latents without a rotated part;
 *      epilogues of the fp32 grouped product; corrected routes, gated joins behind convolutions */
#define PIE_HIP_ABI_VERSION 7
int pie_hip_abi_version(void);

/* ---- W4A16 ("int4b8", symmetric, group-quantised) ------------------------- */

/*
 * Integer unpack test hook: q[n, k] = ((packed[n, k/8] >> (4*(k%8))) & 0xF) - 8
 * as int8.  Bit-exact statement of the nibble order used everywhere else.
 * Reference: driver/cuda/src/kernels/dequant_wna16.cu:31-36.
 */
int pie_hip_unpack_w4(const uint32_t* packed, int8_t* q, int out_dim, int in_dim,
                      void* stream);

/*
 * w[n, k] = bf16( float(nibble - 8) * float(scale[n, k / group_size]) ).
 * packed: [out_dim, in_dim/8] u32, scale: [out_dim, in_dim/group_size] bf16,
 * out: [out_dim, in_dim] bf16.
 * Reference: launch_dequant_wna16_int4b8_to_bf16,
 * driver/cuda/src/kernels/dequant_wna16.hpp:16-23, dequant_wna16.cu:11-38.
 */
int pie_hip_dequant_w4a16(const uint32_t* packed, const uint16_t* scale_bf16,
                          uint16_t* out_bf16, int out_dim, int in_dim, int group_size,
                          void* stream);

/*
 * Weight-only int4 GEMV/skinny GEMM for decode:
 *   y[m, n] = bf16( beta*y[m, n] + sum_k act[m, k] * (nibble(n, k) - 8) * scale[n, k/G] )
 * with fp32 accumulation; the group scale is applied to each group's partial
 * sum (same value as the reference's per-element `x * (q * s)` up to fp32
 * rounding, driver/cuda/src/kernels/dequant_wna16.cu:96-110).
 * Requires K % 32 == 0, G % 32 == 0, K % G == 0.  Tuned for decode (small M): up to four
 * activation rows share one pass over the weights, larger M re-streams them per group of four.
 * Replaces the Marlin call `marlin_w4a16_gemm` for small M
 * (driver/cuda/third_party/marlin/marlin_wrapper.hpp:39-51) and the
 * dequant-then-GEMM fallback of gemm_act_x_w (driver/cuda/src/ops/gemm.cpp:1414-1583).
 */
int pie_hip_gemv_w4a16(const uint16_t* act_bf16, const uint32_t* packed,
                       const uint16_t* scale_bf16, uint16_t* y_bf16, int M, int N, int K,
                       int group_size, int beta, void* stream);
/* Same contract with explicit tiling (rows walked per wave step, resident waves per SIMD;
 * 0 = library default).  For tuning sweeps; no reference counterpart. */
int pie_hip_gemv_w4a16_tuned(const uint16_t* act_bf16, const uint32_t* packed,
                             const uint16_t* scale_bf16, uint16_t* y_bf16, int M, int N, int K,
                             int group_size, int beta, int rows_per_wave, int waves_per_simd,
                             void* stream);

/*
 * The decoder layer's fused projection: y = epilogue( rmsnorm?(act) · W^T ) in one kernel.
 *   norm_weight_bf16 != NULL: act is replaced, while it is staged, by
 *     bf16(act * rsqrt(mean(act^2) + eps) * norm_weight) — value and rounding of the separate
 *     RMSNorm kernel (driver/cuda/src/kernels/rmsnorm.cu:14-54), so results do not change;
 *   swiglu != 0: W's rows are interleaved (gate_0, up_0, gate_1, up_1, ...) and
 *     y[m, i] = bf16( silu(bf16(g_i)) * bf16(u_i) ), y is [M, N/2] — the values of the unfused
 *     projection followed by swiglu_bf16_kernel (driver/cuda/src/kernels/swiglu.cu:9-22);
 *     not combinable with beta.
 * format: PIE_HIP_FMT_*; scale: int4b8 bf16 [N, K/G]; int8/fp8 row scale [N] (f32, or bf16
 * when scale_is_bf16); bf16: NULL.  Other arguments as the per-format GEMV entry points.
 * Replaces the rmsnorm -> gemm_act_x_w (-> swiglu) sequences of
 * driver/cuda/src/model/llama_like.cpp:370-705.
 */
/* Epilogue codes, the `swiglu` argument of every linear entry point: PIE_HIP_EPI_RELU2 stores
 * y[m, n] = bf16( max(sum, 0)^2 ), PIE_HIP_EPI_GELU bf16( sum/2 (1 + erf(sum / sqrt 2)) ) (all N columns;
 * not combinable with beta; GELU over bf16 weights only). */
#define PIE_HIP_EPI_NONE 0
#define PIE_HIP_EPI_SWIGLU 1
#define PIE_HIP_EPI_RELU2 2
#define PIE_HIP_EPI_GELU 3
/* What a gated product (PIE_HIP_EPI_SWIGLU) does with its column pairs besides the plain rule:
 *   g = min(g + bias, limit), u = clamp(u + bias, -limit, limit),
 *   y = g / (1 + exp(-alpha g)) * (u + shift)
 * bias: fp32 [N] in the order of the weight rows (NULL: none), added to the fp32 sums before they are
 * rounded to the output type.  {NULL, INFINITY, 1, 0} is the plain rule. */
typedef struct {
    const float* bias;
    float limit, alpha, shift;
} PieHipGlu;
#define PIE_HIP_FMT_INT4B8 0
#define PIE_HIP_FMT_INT8 1
#define PIE_HIP_FMT_FP8 2
#define PIE_HIP_FMT_BF16 3
int pie_hip_linear_fused(int format, const uint16_t* act_bf16, const uint16_t* norm_weight_bf16,
                         float eps, const void* weight, const void* scale, int scale_is_bf16,
                         int group_size, uint16_t* y_bf16, int M, int N, int K, int beta,
                         int swiglu, void* stream);
/* The same with `glu` (NULL: the plain rule), PIE_HIP_EPI_SWIGLU only. */
int pie_hip_linear_fused_glu(int format, const uint16_t* act_bf16, const uint16_t* norm_weight_bf16,
                             float eps, const void* weight, const void* scale, int scale_is_bf16,
                             int group_size, uint16_t* y_bf16, int M, int N, int K, int beta,
                             int swiglu, const PieHipGlu* glu, void* stream);

/*
 * The attention output projection of a decode step with the attention's split merge in its
 * prologue: y[m, :] = bf16( (beta ? y[m, :] : 0) + o[m, :] . W^T ), where o[m, :] (K = num_q_heads *
 * head_dim values) is the merged, normalised, bf16-rounded attention output of row m — computed
 * from the partial results pie_hip_attn_rows_paged_partials left in attn_workspace with the
 * operations of the separate merge launch in the same order, so y is bit-identical to
 * pie_hip_attn_rows_paged followed by pie_hip_linear_fused.  One launch less per layer: the merge
 * hides behind the projection's first weight requests.  num_splits / units_per_split: the plan
 * pie_hip_attn_decode_plan gave for the same (num_rows = M, num_kv_heads, max_kv_len).  Takes one
 * row with up to eight splits or two rows with up to four, K <= 4096, head_dim a power of two;
 * otherwise PIE_HIP_ERR_UNSUPPORTED (then run pie_hip_attn_rows_paged and pie_hip_linear_fused).
 * Reference: the split-KV merge of the decode attention (attention_flashinfer.hpp:17-24 plans it,
 * the library merges) followed by the o_proj gemm of driver/cuda/src/model/llama_like.cpp:370-705.
 */
int pie_hip_linear_attn_merge_supported(int format, int M, int num_splits, int num_q_heads, int head_dim,
                                        int group_size);   /* 1: taken, 0: PIE_HIP_ERR_UNSUPPORTED */
int pie_hip_linear_attn_merge(int format, const void* attn_workspace, int num_splits, int units_per_split,
                              const int32_t* row_kv_len, int num_q_heads, int head_dim, const void* weight,
                              const void* scale, int scale_is_bf16, int group_size, uint16_t* y_bf16, int M,
                              int N, int beta, void* stream);

/*
 * The fused q|k|v projection of a decode step with RoPE and the KV-cache write in its epilogue:
 * rows of W are the q, k and v heads ([(hq + 2 hk) * d, K]); adjacent output pairs (2i, 2i+1)
 * of every q and k head are rotated by rope_table[m] (interleaved pairing,
 * driver/cuda/src/kernels/rope.cu:14-33), q goes to q_out [M, hq*d], k and v to slot
 * kv_slots[m] of the paged pools (NHD addressing, driver/cuda/src/kernels/split_packed.cu:116-138).
 * Values are those of pie_hip_linear_fused followed by pie_hip_qkv_rope_kvwrite with
 * interleaved = pairing and no q/k norm (every intermediate rounded to bf16 at the same points).
 * pairing = PIE_HIP_ROPE_ADJACENT: as described.  pairing = PIE_HIP_ROPE_HALF_PAIRED_ROWS: the
 * half-split pairing of Llama / Qwen checkpoints (i, i + d/2; driver/cuda/src/kernels/rope.cu:10-21)
 * over weights whose q / k rows were re-ordered at load so that rows (2i, 2i+1) of a head are
 * that pair; the rotated values are written to positions i and i + d/2, so q_out and the pools
 * hold what the unpermuted projection followed by half-split RoPE gives, bit for bit.
 * Replaces the qkv gemm + qkv_decode_qk_norm_rope_write_kv_kernel pair of
 * driver/cuda/src/model/llama_like.cpp:370-470 for llama-type decode.  head_dim a power of two,
 * M <= 4 per weight pass like the GEMV.
 */
int pie_hip_qkv_rope_fused(int format, const uint16_t* act_bf16, const uint16_t* norm_weight_bf16,
                           float eps, const void* weight, const void* scale, int scale_is_bf16,
                           int group_size, int M, int K, const float* rope_table,
                           const int64_t* kv_slots, uint16_t* q_out, uint16_t* k_pages,
                           uint16_t* v_pages, int num_q_heads, int num_kv_heads, int head_dim,
                           int pairing, void* stream);

/*
 * lm_head for greedy decode rows: logits[m, v] = bf16( rmsnorm?(act[m]) . W[v] ) for the bf16
 * matrix W [V, H], and out_tokens[m] = argmax_v logits[m, v] over the bf16 values (the lowest
 * index among equals, NaN never wins, an all -inf row gives 0) — pie_hip_linear_fused followed by
 * pie_hip_argmax, bit for bit, in two launches that read the logits row only once: the GEMV
 * keeps per-lane (largest value, row) pairs while it stores, a one-block-per-row kernel reduces
 * them.  M <= 4 (one pass over the weights); workspace of
 * pie_hip_lm_head_argmax_workspace_bytes(M, V) bytes, need not be cleared.
 * Reference: lm_head_gemv_argmax_bf16 / _int8 (partial (value, index) pairs per block, then a
 * reduce), driver/cuda/src/kernels/argmax.cu:795-935.
 */
size_t pie_hip_lm_head_argmax_workspace_bytes(int M, int V);
int pie_hip_lm_head_argmax(const uint16_t* act_bf16, const uint16_t* norm_weight_bf16, float eps,
                           const uint16_t* w_bf16, uint16_t* logits_bf16, uint32_t* out_tokens, int M,
                           int V, int H, void* workspace, size_t workspace_bytes, void* stream);

/*
 * Weight-only GEMM for a handful to a few dozen activation rows on the matrix cores:
 *   y[m, n] = epilogue( sum_k act[m,k] * w(n,k) ), same formats, scales, beta and swiglu
 * contracts as pie_hip_linear_fused (no fused norm); the weights are streamed once per 16
 * activation rows instead of once per 4.  bf16 products, fp32 accumulation; int4/int8 weights
 * enter the MFMA offset-binary (128+nibble / 128+byte, exact in bf16) and the offset is removed
 * per group / per row in fp32, so the result differs from the GEMV only by fp32 summation order.
 * Requirements (else PIE_HIP_ERR_UNSUPPORTED): K % 512 == 0 and group_size = 128 * 2^i dividing
 * K (int4b8); K % 256 == 0 (int8, fp8); K % 128 == 0 (bf16).
 * Replaces Marlin W4A16 for small/medium M (driver/cuda/third_party/marlin/marlin_wrapper.hpp:39-51)
 * and the cuBLASLt small-M path of gemm_act_x_w (driver/cuda/src/ops/gemm.cpp:1414-1583).
 */
int pie_hip_gemm_skinny(int format, const uint16_t* act_bf16, const void* weight,
                        const void* scale, int scale_is_bf16, int group_size, uint16_t* y_bf16,
                        int M, int N, int K, int beta, int swiglu, void* stream);
/* The same with `glu` (NULL: the plain rule), over row-major or (`tiled`) tile-major weights. */
int pie_hip_gemm_skinny_glu(int format, const uint16_t* act_bf16, const void* weight,
                            const void* scale, int scale_is_bf16, int group_size, uint16_t* y_bf16,
                            int M, int N, int K, int beta, int swiglu, int tiled, const PieHipGlu* glu,
                            void* stream);

/*
 * Tiled weight-only GEMM on the matrix cores for prefill and large batches (compute-bound M):
 *   y[M, N] = epilogue( act[M, K] · W[N, K]^T ), formats / scales / beta / swiglu as above.
 * Evaluation order of the reference's large-M paths: the weights become bf16 first — int4b8 as
 * bf16((nibble-8) * group_scale), the value of launch_dequant_wna16_int4b8_to_bf16
 * (driver/cuda/src/kernels/dequant_wna16.cu:11-38) followed by a bf16 GEMM
 * (driver/cuda/src/ops/gemm.cpp:1213-1236); int8 / fp8 values are exact in bf16 and their row
 * scale multiplies the fp32 sum — then bf16 x bf16 products, fp32 accumulation, one rounding.
 * 128 x 128 x 64 tiles (64 x 128 for M <= 64, 256 x 128 for bf16 weights at large M),
 * v_mfma_f32_16x16x32_bf16.  Requirements: K % 64 == 0; int4b8
 * group_size a power of two >= 32 dividing K.
 */
int pie_hip_gemm_mfma(int format, const uint16_t* act_bf16, const void* weight, const void* scale,
                      int scale_is_bf16, int group_size, uint16_t* y_bf16, int M, int N, int K,
                      int beta, int swiglu, void* stream);

/*
 * The same GEMM for a decode batch (M <= 128 rows), where the output has too few 128-column
 * tiles to fill the machine: K is split into shares, one block per (tile, share), fp32 partial
 * sums go to `workspace` and a second kernel adds them and applies beta / swiglu.  Same
 * evaluation order per share; the shares are added in fp32 in ascending K.
 * pie_hip_gemm_mfma_workspace_bytes(M, N, K) is the workspace this shape needs (0: the shape is
 * not split and the call is pie_hip_gemm_mfma).  Role in the reference: cuBLASLt's split-K
 * heuristics inside gemm_act_x_w for small M (driver/cuda/src/ops/gemm.cpp:1414-1583).
 */
size_t pie_hip_gemm_mfma_workspace_bytes(int M, int N, int K);
int pie_hip_gemm_mfma_splitk(int format, const uint16_t* act_bf16, const void* weight,
                             const void* scale, int scale_is_bf16, int group_size,
                             uint16_t* y_bf16, int M, int N, int K, int beta, int swiglu,
                             void* workspace, size_t workspace_bytes, void* stream);
/* Either of the two (workspace NULL: not split) with `glu` (NULL: the plain rule). */
int pie_hip_gemm_mfma_glu(int format, const uint16_t* act_bf16, const void* weight,
                          const void* scale, int scale_is_bf16, int group_size,
                          uint16_t* y_bf16, int M, int N, int K, int beta, int swiglu,
                          const PieHipGlu* glu, void* workspace, size_t workspace_bytes, void* stream);

/*
 * MoE grouped weight-only GEMM: one skinny problem per expert in a single launch.
 *   rows [expert_offsets[e], expert_offsets[e+1]) of y (routes sorted by expert) are
 *   act[route_act_rows[r]] (or act[r] when route_act_rows is NULL) times expert e's [N,K]
 *   weights at weights + e*weight_stride_bytes (scales at scales + e*scale_stride_bytes).
 * Experts without routes cost nothing and their weights are never read; an expert's weights
 * are read once per 16 routes that hit it.  max_rows_per_expert is a hint (> 0) of the largest
 * per-expert row count; num_routes (0: not known) bounds how many experts have any.  With swiglu the weight rows are interleaved (gate_0, up_0, ...) and y
 * is [routes, N/2].  Same K requirements as pie_hip_gemm_skinny.
 * Replaces the per-route MoE decode GEMVs (driver/cuda/src/kernels/dequant_wna16.cu:59-169)
 * and the grouped GEMM of driver/cuda/src/ops/gemm.hpp:189-198.
 */
int pie_hip_moe_grouped_gemm(int format, const uint16_t* act_bf16, const int32_t* route_act_rows,
                             const int32_t* expert_offsets, int num_experts,
                             int max_rows_per_expert, const void* weights,
                             size_t weight_stride_bytes, const void* scales,
                             size_t scale_stride_bytes, int scale_is_bf16, int group_size,
                             uint16_t* y_bf16, int N, int K, int swiglu, void* stream);
/* The same with `glu` (NULL: the plain rule; its bias is [N], the same for every expert), over row-major or
 * (`tiled`) tile-major weights. */
int pie_hip_moe_grouped_gemm_glu(int format, const uint16_t* act_bf16, const int32_t* route_act_rows,
                                 const int32_t* expert_offsets, int num_experts,
                                 int max_rows_per_expert, int num_routes, const void* weights,
                                 size_t weight_stride_bytes, const void* scales,
                                 size_t scale_stride_bytes, int scale_is_bf16, int group_size,
                                 uint16_t* y_bf16, int N, int K, int swiglu, int tiled,
                                 const PieHipGlu* glu, void* stream);
/* bf16 experts with many routes each (a prompt's tokens): the tiled GEMM's blocks of block_rows (64, 128, 256; 0:
 * chosen from the routes per expert) routes of one expert, whose weights are read once per block.  num_routes =
 * expert_offsets[num_experts].  K % 64 == 0, tile-major weights need N % 16 == 0. */
int pie_hip_moe_grouped_gemm_mfma(const uint16_t* act_bf16, const int32_t* route_act_rows, const int32_t* expert_offsets,
                                  int num_experts, int num_routes, const void* weights_bf16, size_t weight_stride_bytes,
                                  uint16_t* y_bf16, int N, int K, int epilogue, int tiled, const PieHipGlu* glu,
                                  int block_rows, void* stream);

/*
 * Tile-major weight layout for the skinny and grouped GEMMs.  The 16 bytes that lane (j, q) of a
 * wave loads for the 16-row tile t and K block b — byte 64 b + 16 q of row 16 t + j in the
 * row-major [N, K] matrix — are stored at byte ((t * nb + b) * 64 + 16 q + j) * 16, nb =
 * row_bytes / 64, so every wave load is 1 KiB contiguous instead of 16 rows x 64 bytes (rows past
 * N are zero; dst holds ceil(N/16) * 16 * row_bytes bytes).  int4 group scales [N, groups] become
 * [tile][group][16 rows].  Built once at load; the values are those of the row-major entry
 * points.  int4b8 weights take pie_hip_repack_mfma_tiles_int4, which also re-orders the eight
 * codes of every 32-bit word (codes 2i and 2i + 1 to nibbles i and i + 4) so that the kernels'
 * decode yields them in k order; the other formats take pie_hip_repack_mfma_tiles.  Role in the
 * reference: Marlin's offline weight repack (driver/cuda/third_party/marlin/marlin_wrapper.hpp:39-51).
 */
int pie_hip_repack_mfma_tiles(const void* src, void* dst, int N, size_t row_bytes, void* stream);
int pie_hip_repack_mfma_tiles_int4(const void* src, void* dst, int N, size_t row_bytes, void* stream);
int pie_hip_repack_scale_tiles(const uint16_t* src, uint16_t* dst, int N, int groups, void* stream);
/* pie_hip_gemm_skinny / pie_hip_moe_grouped_gemm over weights (and int4 group scales) in that
 * layout; every other argument as there (expert strides in bytes of the tiled buffers). */
int pie_hip_gemm_skinny_tiled(int format, const uint16_t* act_bf16, const void* weight,
                        const void* scale, int scale_is_bf16, int group_size, uint16_t* y_bf16,
                        int M, int N, int K, int beta, int swiglu, void* stream);
/* pie_hip_qkv_rope_fused for more rows than the GEMV takes (a decode batch): the q|k|v projection
 * over tile-major weights with interleaved RoPE and the KV-cache write in its epilogue.  act_bf16
 * is the normalised activation [M, K]; values are those of pie_hip_gemm_skinny_tiled followed by
 * pie_hip_qkv_rope_kvwrite (interleaved = pairing, 1 or 2; no q/k norm), every intermediate rounded to bf16 at
 * the same points.  Same reference role: the qkv gemm + qkv_decode_qk_norm_rope_write_kv_kernel
 * pair of driver/cuda/src/model/llama_like.cpp:370-470.  head_dim a power of two, K % 256 == 0. */
int pie_hip_qkv_rope_skinny_tiled(int format, const uint16_t* act_bf16, const void* weight,
                                  const void* scale, int scale_is_bf16, int group_size, int M, int K,
                                  const float* rope_table, const int64_t* kv_slots, uint16_t* q_out,
                                  uint16_t* k_pages, uint16_t* v_pages, int num_q_heads,
                                  int num_kv_heads, int head_dim, int pairing, void* stream);
int pie_hip_moe_grouped_gemm_tiled(int format, const uint16_t* act_bf16, const int32_t* route_act_rows,
                             const int32_t* expert_offsets, int num_experts,
                             int max_rows_per_expert, const void* weights,
                             size_t weight_stride_bytes, const void* scales,
                             size_t scale_stride_bytes, int scale_is_bf16, int group_size,
                             uint16_t* y_bf16, int N, int K, int swiglu, void* stream);

/*
 * MoE routing: per token softmax over router_logits[t, 0..E) (bf16 in, fp32 inside), top_k by
 * repeated argmax with exclusion (ties to the lowest expert index), weights renormalised to
 * sum 1 — topk_softmax_bf16_kernel, driver/cuda/src/kernels/topk_softmax.cu:19-86 (graph form:
 * driver/portable/src/graph_common.cpp:262-283).  A second small kernel builds the grouped layout of
 * pie_hip_moe_grouped_gemm: routes (t, k) counting-sorted by expert.
 *   topk_idx [T, top_k] int32, topk_weight [T, top_k] f32 (bit-exact integer outputs given the
 *   probabilities; the order of routes inside one expert is unspecified),
 *   expert_offsets [E+1], route_token [T*top_k] (token of each sorted route),
 *   route_pos [T*top_k] (sorted position of route (t, k)).
 * num_experts <= 512, top_k <= 16 (the reference's bounds).
 * pie_hip_moe_route_opt: renormalize = 0 leaves the chosen experts' softmax probabilities undivided
 * (norm_topk = false: the graph form divides only under it, graph_common.cpp:279-283);
 * pie_hip_moe_route is renormalize = 1.
 */
int pie_hip_moe_route(const uint16_t* router_logits_bf16, int32_t* topk_idx, float* topk_weight,
                      int32_t* expert_offsets, int32_t* route_token, int32_t* route_pos,
                      int num_tokens, int num_experts, int top_k, void* stream);
int pie_hip_moe_route_opt(const uint16_t* router_logits_bf16, int32_t* topk_idx, float* topk_weight,
                      int32_t* expert_offsets, int32_t* route_token, int32_t* route_pos,
                      int num_tokens, int num_experts, int top_k, int renormalize, void* stream);
/* The same from fp32 logits (rows of ld_logits), with the experts in num_groups equal groups of neighbours:
 * a token chooses among the experts of the keep_groups groups whose best expert has the largest probability
 * (ties to the lowest group); weight = p / (sum of the chosen p + 1e-20) * weight_scale.  top_k <= 64 and at most
 * keep_groups * num_experts / num_groups.  Up to sixteen tokens take one launch. */
int pie_hip_moe_route_groups(const float* router_logits, int ld_logits, int32_t* topk_idx, float* topk_weight,
                             int32_t* expert_offsets, int32_t* route_token, int32_t* route_pos, int num_tokens,
                             int num_experts, int top_k, int num_groups, int keep_groups, float weight_scale,
                             void* stream);

/*
 * A decode batch's way into the MoE block in two launches instead of four: per token the RMSNorm
 * of its hidden row (norm_out = what pie_hip_rmsnorm stores, bit for bit), the router logits
 * bf16(sum_k norm_out[t, k] * router[e, k]) over the bf16 router matrix [E, hidden] (fp32 sums in
 * this kernel's own order: they may differ from a GEMM's in the last bf16 bit), pie_hip_moe_route_opt's
 * softmax / top-k on them, then the expert-sorted layout.  router_logits may be NULL (not stored).
 * Each token's block reads the whole router matrix through the L2: meant for batches of up to a
 * few hundred rows.  hidden <= 8192, a multiple of 8; expert and top-k bounds as pie_hip_moe_route.
 * Replaces rmsnorm + router gemm + topk_softmax_bf16_kernel of the reference's MoE block
 * (driver/cuda/src/model/kimi_forward.cpp:640-700; graph form driver/portable/src/graph_common.cpp:237-283).
 */
int pie_hip_moe_norm_route(const uint16_t* x_bf16, const uint16_t* norm_weight_bf16, float eps,
                           const uint16_t* router_bf16, uint16_t* norm_out_bf16,
                           uint16_t* router_logits_bf16, int32_t* topk_idx, float* topk_weight,
                           int32_t* expert_offsets, int32_t* route_token, int32_t* route_pos,
                           int num_tokens, int hidden, int num_experts, int top_k, int renormalize,
                           void* stream);

/*
 * pie_hip_moe_combine with add = 1 followed by pie_hip_rmsnorm of the updated rows with the next
 * layer's norm weight, in one launch and with both results bit-identical to the two:
 * out[t, :] = bf16(out[t, :] + sum_k w[t, k] * y_routes[route_pos[t, k], :]),
 * norm_out[t, :] = rmsnorm(out[t, :]) * norm_weight.  hidden <= 8192, a multiple of 8.
 * Reference: token_batched_weighted_sum_add_bf16_kernel (driver/cuda/src/kernels/moe_dispatch.cu:152-196)
 * + rmsnorm_bf16_kernel (driver/cuda/src/kernels/rmsnorm.cu:14-54).
 */
int pie_hip_moe_combine_norm(const uint16_t* y_routes_bf16, const int32_t* route_pos,
                             const float* topk_weight, uint16_t* out_bf16,
                             const uint16_t* norm_weight_bf16, float eps, uint16_t* norm_out_bf16,
                             int num_tokens, int top_k, int hidden, void* stream);

/*
 * MoE combine: out[t, :] = bf16( (add ? out[t, :] : 0) + sum_k topk_weight[t, k] *
 * y_routes[route_pos[t, k], :] ), fp32 sum in top-k order, one rounding —
 * token_batched_weighted_sum[_add]_bf16_kernel, driver/cuda/src/kernels/moe_dispatch.cu:152-196.
 * hidden % 8 == 0.
 */
int pie_hip_moe_combine(const uint16_t* y_routes_bf16, const int32_t* route_pos,
                        const float* topk_weight, uint16_t* out_bf16, int num_tokens, int top_k,
                        int hidden, int add, void* stream);

/*
 * Prefill attention on the matrix cores: the result contract of pie_hip_attn_rows_paged for
 * query rows grouped into tiles.  Tile i covers rows tile_row_start[i] .. + tile_num_rows[i]
 * (consecutive rows that share one page list, i.e. row_page_begin is equal across the tile;
 * at most rows_per_tile rows, which is pie_hip_attn_prefill_tile_rows(hq, hk) = 128 / (hq/hk)
 * or half of it — the smaller tile doubles the number of blocks for small batches); each row
 * still sees its own first row_kv_len[row] keys.  Tiles may come in any order; blocks start in tile
 * order (the kv heads of a tile side by side), so listing the tiles with the longest key extents
 * first lets the short ones fill the slots that free up — on a causal prompt of more tiles than the
 * device holds at once that is worth 15-30 % (4096 tokens: 355 -> 278 us).  Probabilities are rounded to bf16 before they multiply V
 * (fp32 softmax sums and accumulators), so results agree with the per-row kernel to about one
 * bf16 step rather than bit for bit.  d in {64,128}, hq/hk in {1,2,4,8}, page_size % 16 == 0.
 * Reference: the causal prefill branch of launch_attention_naive_paged_prefill,
 * driver/cuda/src/ops/attention_naive_paged.cu:148-317; per-request flash attention of the
 * portable driver, driver/portable/src/graph_common.cpp:347-396.
 */
int pie_hip_attn_prefill_tile_rows(int num_q_heads, int num_kv_heads);
int pie_hip_attn_prefill_tiles(const uint16_t* q, const uint16_t* k_pages, const uint16_t* v_pages,
                               uint16_t* o, const uint32_t* kv_page_indices,
                               const uint32_t* row_page_begin, const int32_t* row_kv_len,
                               const int32_t* tile_row_start, const int32_t* tile_num_rows,
                               int num_tiles, int rows_per_tile, int num_q_heads, int num_kv_heads,
                               int head_dim, int page_size, float sm_scale, void* stream);
/* The same over one-byte KV pools (kv_format / k_scales / v_scales as for
 * pie_hip_attn_rows_paged_kvq; PIE_HIP_KV_BF16 with null scales is pie_hip_attn_prefill_tiles):
 * codes are decoded exactly into the bf16 tiles, the K scale multiplies the score and the V
 * scale the rounded probability. */
int pie_hip_attn_prefill_tiles_kvq(int kv_format, const uint16_t* q, const void* k_pages,
                                   const void* v_pages, const float* k_scales, const float* v_scales,
                                   uint16_t* o, const uint32_t* kv_page_indices,
                                   const uint32_t* row_page_begin, const int32_t* row_kv_len,
                                   const int32_t* tile_row_start, const int32_t* tile_num_rows,
                                   int num_tiles, int rows_per_tile, int num_q_heads, int num_kv_heads,
                                   int head_dim, int page_size, float sm_scale, void* stream);

/*
 * Custom attention masks for the per-row form.  pie_hip_attn_mask_bitmap turns per-row BRLE
 * runs into one u16 per 16-token unit (bit t = key 16*unit + t visible): run_bounds holds each
 * row's cumulative run ends, [run_bounds_indptr[r], run_bounds_indptr[r+1]); runs alternate
 * hidden / visible from key 0, keys past the last run are hidden, a row without runs sees its
 * whole window; no key at or past row_kv_len[r] (= the row's position + 1) is ever visible, and
 * window > 0 also hides keys below row_kv_len[r] - window
 * (build_attn_mask_f16, driver/portable/src/plan.cpp:54-94).  bitmap: [num_rows, stride_units],
 * stride_units >= ceil(max_kv_len / 16).
 * pie_hip_attn_rows_paged_masked is pie_hip_attn_rows_paged restricted to the visible keys; a
 * row with no visible key gives o = 0, lse = -inf.
 */
int pie_hip_attn_mask_bitmap(const uint32_t* run_bounds, const int32_t* run_bounds_indptr,
                             const int32_t* row_kv_len, int window, uint16_t* bitmap, int num_rows,
                             int stride_units, void* stream);
int pie_hip_attn_rows_paged_masked(const uint16_t* q, const uint16_t* k_pages, const uint16_t* v_pages,
                                   uint16_t* o, float* lse, const uint32_t* kv_page_indices,
                                   const uint32_t* row_page_begin, const int32_t* row_kv_len,
                                   const uint16_t* mask_bitmap, int mask_stride_units, int num_rows,
                                   int num_q_heads, int num_kv_heads, int head_dim, int page_size,
                                   float sm_scale, int max_kv_len, void* workspace,
                                   size_t workspace_bytes, void* stream);

/*
 * Sampling beyond greedy argmax, one slot = one sampled logits row.
 *
 * pie_hip_sample_gather_logits: out[s, :] = f32(logits[rows[s], :]) (rows == NULL: row s), with
 * slot s's BRLE logit mask applied: mask_bounds[mask_bounds_indptr[s] .. [s+1]) are the
 * cumulative ends of the slot's runs; run j (0-based) allows its tokens when j is odd, tokens
 * past the last run are masked (-inf), a slot with no runs is unconstrained
 * (apply_brle_logit_mask, driver/portable/src/sampler.cpp:169-198).
 *
 * pie_hip_sample: per slot, by `kind` (the wire order of the Sampler variants,
 * driver/bridge/include/pie_bridge/view.hpp:346-358):
 *   MULTINOMIAL / TOP_K / TOP_P / MIN_P / TOP_K_TOP_P -> tokens[s]
 *       (sample_token, driver/portable/src/sampler.cpp:345-409; uniform[s] is the draw the
 *       reference takes from its per-slot PCG32, made by the caller)
 *   DIST      -> ids / values [out_indptr[s], out_indptr[s+1]): the most probable tokens of
 *                softmax(logits / T), descending (run_distribution, :224-251); the range length
 *                is the caller's k (the whole vocabulary for k = 0)
 *   LOGPROB / LOGPROBS -> values[i] = log_softmax(logits)[labels[i]] over the slot's range
 *                (run_logprob / run_logprobs_many, :262-292); labels must be < vocab
 *   ENTROPY   -> values[out_indptr[s]] (run_entropy, :294-306)
 *   RAW_LOGITS -> nothing: the f32 row of pie_hip_sample_gather_logits is the payload
 * Equal probabilities are ordered by ascending token id.  Running sums are taken in double and
 * compared after rounding to float.  workspace: pie_hip_sample_workspace_bytes(S, vocab).
 */
enum {
    PIE_HIP_SAMPLER_MULTINOMIAL = 0, PIE_HIP_SAMPLER_TOP_K = 1, PIE_HIP_SAMPLER_TOP_P = 2,
    PIE_HIP_SAMPLER_MIN_P = 3, PIE_HIP_SAMPLER_TOP_K_TOP_P = 4,
    PIE_HIP_SAMPLER_EMBEDDING = 5,   /* a slot without output (the reference's executor emits nothing for it) */
    PIE_HIP_SAMPLER_DIST = 6,
    PIE_HIP_SAMPLER_RAW_LOGITS = 7, PIE_HIP_SAMPLER_LOGPROB = 8, PIE_HIP_SAMPLER_LOGPROBS = 9,
    PIE_HIP_SAMPLER_ENTROPY = 10
};
size_t pie_hip_sample_workspace_bytes(int num_slots, int vocab);
int pie_hip_sample_gather_logits(const uint16_t* logits_bf16, const int32_t* rows, float* out_f32,
                                 const uint32_t* mask_bounds, const int32_t* mask_bounds_indptr,
                                 int num_slots, int vocab, void* stream);
int pie_hip_sample(const float* logits_f32, const int32_t* kind, const float* temperature,
                   const uint32_t* top_k, const float* top_p, const float* min_p,
                   const float* uniform, const int32_t* out_indptr, const uint32_t* labels,
                   uint32_t* tokens, float* values, uint32_t* ids, void* workspace,
                   size_t workspace_bytes, int num_slots, int vocab, void* stream);

/* Measurement form of pie_hip_gemv_w4a16 (M <= 4: one kernel): that kernel is bracketed by the
 * caller's two HIP events (hipEvent_t), so hipEventElapsedTime(start, stop) is its own duration.
 * The events belong to this call only; the library keeps nothing.  No reference counterpart. */
int pie_hip_gemv_w4a16_timed(const uint16_t* act_bf16, const uint32_t* packed,
                             const uint16_t* scale_bf16, uint16_t* y_bf16, int M, int N, int K,
                             int group_size, int beta, void* start_event, void* stop_event,
                             void* stream);

/*
 * Weight-only int8 GEMV (W8A16), per-output-channel scale:
 *   y[m, n] = bf16( beta*y[m, n] + (sum_k f32(act[m,k]) * f32(q[n,k])) * scale_inv[n] )
 * fp32 sum, scale applied once after it — the evaluation order of the reference's own
 * weight-only int8 GEMV (driver/cuda/src/kernels/argmax.cu:846-854).  q: int8 [N,K];
 * scale_inv (= absmax/127, driver/cuda/src/kernels/quant_bf16_to_fp8.cu:311-313) is given
 * as f32 [N] or as bf16 [N]: pass exactly one of the two pointers.  K % 16 == 0.
 */
int pie_hip_gemv_w8a16(const uint16_t* act_bf16, const int8_t* w_int8,
                       const float* scale_inv_f32, const uint16_t* scale_inv_bf16,
                       uint16_t* y_bf16, int M, int N, int K, int beta, void* stream);

/*
 * Weight-only fp8 (OCP e4m3fn bytes) GEMV with per-output-channel scale, same shape rules
 * and scale arguments as the int8 entry point.  Format:
 * driver/cuda/src/kernels/dequant_fp8.cu:25-39 (w = fp8 * scale_inv[row]).
 */
int pie_hip_gemv_fp8(const uint16_t* act_bf16, const uint8_t* w_e4m3,
                     const float* scale_inv_f32, const uint16_t* scale_inv_bf16,
                     uint16_t* y_bf16, int M, int N, int K, int beta, void* stream);

/*
 * bf16 GEMV: y[m, n] = bf16( beta*y + sum_k act[m,k]*W[n,k] ), fp32 accumulation
 * (gemm_act_x_w bf16 path, driver/cuda/src/ops/gemm.hpp:152-160; the lm_head and router
 * projections stay unquantised in the reference).  K % 8 == 0.
 */
int pie_hip_gemv_bf16(const uint16_t* act_bf16, const uint16_t* w_bf16, uint16_t* y_bf16, int M,
                      int N, int K, int beta, void* stream);

/* ---- paged-KV decode attention -------------------------------------------- */

/*
 * One query token per request over a paged KV pool:
 *   o[r, h, :] = softmax_j( q[r,h,:]·K[j, kvh, :] * sm_scale ) · V[j, kvh, :],  kvh = h / (hq/hk)
 * for j over the request's context, kv_len = (pages-1)*page_size + last_page_len
 * (0 when the request lists no page; then o = 0 and lse = -inf).
 *   q, o          [R, hq, d] bf16
 *   k_pages/v_pages [num_pages, page_size, hk, d] bf16 (driver/cuda/src/kv_cache.hpp:3-8)
 *   kv_page_indices / kv_page_indptr[R+1] / kv_last_page_lens[R]: the wire arrays of
 *     the forward request, as the runtime sends them; requests may list the same
 *     physical pages (forked prefixes) — they are read in place.
 *   lse           optional [R, hq] f32, natural-log sum-exp of the scaled scores
 *   sm_scale      <= 0 selects 1/sqrt(d)
 *   max_kv_len    host-side upper bound on any request's kv_len (sizes the split grid)
 *   workspace     device scratch of pie_hip_attn_decode_workspace_bytes(...) bytes
 * fp32 maths, one bf16 rounding at the output.  d in {64,128}, hq/hk in {1,2,4,8},
 * page_size % 16 == 0.
 * Reference: launch_attention_naive_paged_decode,
 * driver/cuda/src/ops/attention_naive_paged.hpp:57-69, kernel attention_naive_paged.cu:319-447;
 * split-KV planning role of driver/cuda/src/ops/attention_flashinfer.hpp:17-24.
 */
size_t pie_hip_attn_decode_workspace_bytes(int num_requests, int num_q_heads, int num_kv_heads,
                                           int head_dim, int max_kv_len);
int pie_hip_attn_decode_paged(const uint16_t* q, const uint16_t* k_pages, const uint16_t* v_pages,
                              uint16_t* o, float* lse, const uint32_t* kv_page_indices,
                              const uint32_t* kv_page_indptr, const uint32_t* kv_last_page_lens,
                              int num_requests, int num_q_heads, int num_kv_heads, int head_dim,
                              int page_size, float sm_scale, int max_kv_len, void* workspace,
                              size_t workspace_bytes, void* stream);

/*
 * Same attention over explicit per-row extents: query row r reads the page-list entries
 * starting at kv_page_indices[row_page_begin[r]] and sees its first row_kv_len[r] keys.  A
 * planner derives the pairs from the page table and the token positions
 * (visible keys = min(seq_len, position + 1), driver/portable/src/plan.cpp:54-94), so a
 * prefill or mixed batch runs as one row per query token, causal by construction, and a
 * decode batch as one row per request.  Workspace: pie_hip_attn_decode_workspace_bytes with
 * num_requests = num_rows.
 */
/* How a decode attention launch over (num_rows, num_kv_heads, max_kv_len) splits its rows:
 * units_per_split 16-token units per split, num_splits splits per row (1: no workspace, no merge). */
int pie_hip_attn_decode_plan(int num_rows, int num_kv_heads, int max_kv_len, int* units_per_split,
                             int* num_splits);
/* Whether a decode attention launch without custom masks over pools of kv_format takes the chunked
 * form instead of that grid of splits: as many blocks as the device holds at once, each with the same
 * share of the batch's keys (one wave per kv head, the rows' keys in 16-token units cut into equal
 * chunks), for one-byte pools when the grid would queue blocks behind one another.  The workspace
 * query covers both forms; results agree to the rounding of the fp32 merge.  Informational (tests,
 * profiles): 1 or 0. */
int pie_hip_attn_decode_is_chunked(int kv_format, int num_rows, int num_kv_heads, int max_kv_len);
/* pie_hip_attn_rows_paged (kv_format PIE_HIP_KV_BF16) / pie_hip_attn_rows_paged_kvq without the merge
 * launch: the splits' partial results stay in the workspace — [rows, q heads, splits, head_dim] f32
 * unnormalised outputs, then [rows, q heads, splits, 2] f32 (max, sum) in units of scale * log2(e);
 * slots of splits past a row's own extent are left unwritten — for pie_hip_linear_attn_merge.
 * PIE_HIP_ERR_INVALID when the plan has a single split (nothing to merge). */
int pie_hip_attn_rows_paged_partials(int kv_format, const uint16_t* q, const void* k_pages, const void* v_pages,
                                     const float* k_scales, const float* v_scales,
                                     const uint32_t* kv_page_indices, const uint32_t* row_page_begin,
                                     const int32_t* row_kv_len, int num_rows, int num_q_heads,
                                     int num_kv_heads, int head_dim, int page_size, float sm_scale,
                                     int max_kv_len, void* workspace, size_t workspace_bytes, void* stream);
int pie_hip_attn_rows_paged(const uint16_t* q, const uint16_t* k_pages, const uint16_t* v_pages,
                            uint16_t* o, float* lse, const uint32_t* kv_page_indices,
                            const uint32_t* row_page_begin, const int32_t* row_kv_len,
                            int num_rows, int num_q_heads, int num_kv_heads, int head_dim,
                            int page_size, float sm_scale, int max_kv_len, void* workspace,
                            size_t workspace_bytes, void* stream);

/*
 * pie_hip_attn_rows_paged without a workspace argument and without any allocation, for callers
 * that cannot allocate device memory: code running under HIP graph capture, tight serving loops,
 * harnesses that forbid hipMalloc.  It has no counterpart in the reference.  The split partials
 * go to a device array built into the library, PIE_HIP_ATTN_STATIC_SCRATCH_BYTES per GPU, held
 * until the process ends; a batch whose partials
 * (pie_hip_attn_decode_workspace_bytes(num_rows, ...)) exceed it is refused with
 * PIE_HIP_ERR_UNSUPPORTED and a message on stderr.  Same kernels and results as
 * pie_hip_attn_rows_paged, bit for bit.  All calls on one GPU share that GPU's array: calls
 * that overlap on one GPU (different streams, or threads) race; serialise them.  The first call
 * on a device looks up the array's address (no allocation, but make it outside graph capture).
 */
#define PIE_HIP_ATTN_STATIC_SCRATCH_BYTES (16u << 20)
int pie_hip_attn_rows_paged_static(const uint16_t* q, const uint16_t* k_pages,
                                   const uint16_t* v_pages, uint16_t* o, float* lse,
                                   const uint32_t* kv_page_indices, const uint32_t* row_page_begin,
                                   const int32_t* row_kv_len, int num_rows, int num_q_heads,
                                   int num_kv_heads, int head_dim, int page_size, float sm_scale,
                                   int max_kv_len, void* stream);

/*
 * KV-cache storage formats of the pool (the CUDA driver's kv_cache_dtype values,
 * driver/cuda/src/kv_cache_format.cpp:46-110).  One-byte formats keep the bf16 layout
 * [pages, page_size, hk, d] with one byte per element; the per-token-head formats add fp32 side
 * scales [pages, hk, page_size] for K and for V (see pie_hip_kv_write_quant).  The 4-bit block format
 * ("fp4_e2m1" / "nvfp4": the same scheme under two names) packs two e2m1 codes per byte,
 * [pages, page_size, hk, d/2] with the even element in the low nibble, and keeps one fp32 scale
 * per block of 16 elements, [pages, hk, page_size, d/16]; the attention entry points do not read
 * it directly (PIE_HIP_ERR_UNSUPPORTED): as in the reference, the pages a batch reads are first
 * expanded into a bf16 pool by pie_hip_kv_dequant_pages.
 */
enum {
    PIE_HIP_KV_BF16 = 0,
    PIE_HIP_KV_FP8_E4M3 = 1,             /* saturating cast of the value, no scales */
    PIE_HIP_KV_INT8_PER_TOKEN_HEAD = 2,  /* scale = absmax/127, code = rint(x / scale) */
    PIE_HIP_KV_FP8_PER_TOKEN_HEAD = 3,   /* scale = absmax/448, code = e4m3(x / scale) */
    PIE_HIP_KV_FP8_E5M2 = 4,             /* saturating e5m2 cast of the value, no scales */
    PIE_HIP_KV_FP4_BLOCK = 5             /* per 16 elements: scale = absmax/6, code = nearest e2m1 level */
};

/*
 * pie_hip_attn_rows_paged over a pool in a one-byte format: every K / V element is
 * float(code) * scale as load_kv_scalar reads it (driver/cuda/src/ops/attention_naive_paged.cu:56-112),
 * everything else as for bf16 pools.  k_scales / v_scales: required for the per-token-head
 * formats, NULL for PIE_HIP_KV_FP8_E4M3 and PIE_HIP_KV_FP8_E5M2.  Custom masks are not available with these formats.
 */
int pie_hip_attn_rows_paged_kvq(int kv_format, const uint16_t* q, const void* k_pages,
                                const void* v_pages, const float* k_scales, const float* v_scales,
                                uint16_t* o, float* lse, const uint32_t* kv_page_indices,
                                const uint32_t* row_page_begin, const int32_t* row_kv_len,
                                int num_rows, int num_q_heads, int num_kv_heads, int head_dim,
                                int page_size, float sm_scale, int max_kv_len, void* workspace,
                                size_t workspace_bytes, void* stream);
/* The same call (any kv_format, PIE_HIP_KV_BF16 with NULL scales included) for a batch whose rows
 * the caller knows to be about equally long, e.g. a decode batch whose longest context is within an
 * eighth of the mean: the launch then takes one round of resident blocks — for 64 rows of 8 kv
 * heads one block per (row, kv head), nothing to merge — where rows of unknown lengths get several
 * splits so that a long one does not run on alone.  Same results contract and workspace query;
 * a wrong hint costs time, not correctness.  Reference: the decode branch of
 * launch_attention_naive_paged, driver/cuda/src/ops/attention_naive_paged.cu:319-447 (one launch
 * per batch; the split plan is this library's). */
int pie_hip_attn_rows_paged_kvq_uniform(int kv_format, const uint16_t* q, const void* k_pages,
                                        const void* v_pages, const float* k_scales, const float* v_scales,
                                        uint16_t* o, float* lse, const uint32_t* kv_page_indices,
                                        const uint32_t* row_page_begin, const int32_t* row_kv_len,
                                        int num_rows, int num_q_heads, int num_kv_heads, int head_dim,
                                        int page_size, float sm_scale, int max_kv_len, void* workspace,
                                        size_t workspace_bytes, void* stream);
/* The same over rows with custom attention masks: mask_bitmap as for
 * pie_hip_attn_rows_paged_masked (one visibility word per row and 16-token unit). */
int pie_hip_attn_rows_paged_kvq_masked(int kv_format, const uint16_t* q, const void* k_pages,
                                       const void* v_pages, const float* k_scales,
                                       const float* v_scales, uint16_t* o, float* lse,
                                       const uint32_t* kv_page_indices,
                                       const uint32_t* row_page_begin, const int32_t* row_kv_len,
                                       const uint16_t* mask_bitmap, int mask_stride_units,
                                       int num_rows, int num_q_heads, int num_kv_heads, int head_dim,
                                       int page_size, float sm_scale, int max_kv_len,
                                       void* workspace, size_t workspace_bytes, void* stream);

/*
 * Quantising KV write: this step's K and V rows [num_tokens, hk, d] bf16 (after RoPE) go to
 * slot kv_slots[t] of a one-byte pool (slot < 0: skipped).  Per-token-head formats:
 * scale = absmax / qmax (qmax 127 / 448; 1 for an all-zero row), code = x * (1/scale) rounded
 * to nearest even, clamped / saturated; PIE_HIP_KV_FP8_E4M3 / _E5M2: the saturating cast of x
 * (largest finite value 448 / 57344).  The fp32 scale pools are laid out
 * [pages, kv heads, page_size] (the 16 scales an attention block reads for one page and head are
 * contiguous; a page's scales are one run, so page copies move them like the codes): the scale of
 * slot s and head h sits at ((s / page_size) * hk + h) * page_size + s % page_size.
 * Reference: write_kv_per_token_head_kernel and write_kv_fp8_per_tensor_kernel,
 * driver/cuda/src/kernels/kv_paged.cu:155-297.
 */
int pie_hip_kv_write_quant(int kv_format, const uint16_t* k_rows, const uint16_t* v_rows,
                           const int64_t* kv_slots, void* k_pages, void* v_pages, float* k_scales,
                           float* v_scales, int num_tokens, int num_kv_heads, int head_dim,
                           int page_size, void* stream);
/* PIE_HIP_KV_FP4_BLOCK in pie_hip_kv_write_quant: per block of 16 elements scale = absmax / 6
 * (1 for an all-zero block), code = the nearest of +-{0, .5, 1, 1.5, 2, 3, 4, 6} to x * (1/scale),
 * the smaller magnitude on a tie, sign bit for x < 0 (write_kv_fp4_block_kernel,
 * driver/cuda/src/kernels/kv_paged.cu:292-417); head_dim a multiple of 16.
 *
 * Expansion of the pages a batch reads into bf16 pools of the same geometry
 * [pages, page_size, hk, d] (page ids unchanged; other pages are not touched): every element
 * becomes bf16(float(code) * scale), for any of the one-byte formats and the 4-bit block format.
 * page_ids may name a page more than once.
 * Reference: launch_dequant_kv_cache_layer_to_bf16_active and the dequant_*_pages_active kernels,
 * driver/cuda/src/kernels/kv_paged.cu:419-531, :698-770. */
int pie_hip_kv_dequant_pages(int kv_format, const void* k_pages, const void* v_pages,
                             const float* k_scales, const float* v_scales, uint16_t* k_out,
                             uint16_t* v_out, const uint32_t* page_ids, int num_pages,
                             int num_kv_heads, int head_dim, int page_size, void* stream);
/* pie_hip_qkv_rope_kvwrite and pie_hip_kv_write_quant in one launch for one-byte pools: every
 * (token, head) of the packed q|k|v rows is rotated (optional per-head q/k RMSNorm, either
 * pairing) and rounded to bf16 as by pie_hip_qkv_rope_kvwrite; q goes to q_out, the K and V
 * heads are quantised from those bf16 values into the token's slot with the arithmetic of
 * pie_hip_kv_write_quant (driver/cuda/src/kernels/kv_paged.cu:155-297) — the same bytes and
 * scales as the two calls in a row.  head_dim <= 256. */
int pie_hip_qkv_rope_kvwrite_quant(int kv_format, const uint16_t* packed_qkv, uint16_t* q_out,
                                   void* k_pages, void* v_pages, float* k_scales, float* v_scales,
                                   const uint16_t* q_norm_weight, const uint16_t* k_norm_weight,
                                   const float* rope_table, const int64_t* kv_slots, int num_tokens,
                                   int num_q_heads, int num_kv_heads, int head_dim, int page_size,
                                   int interleaved, float eps, void* stream);

/* ---- per-layer kernels of the llama-like decoder ---------------------------- */

/* y[n,:] = table[token_ids[n],:]; ids >= vocab read row 0.
 * Reference: launch_embed_bf16, driver/cuda/src/kernels/embed.cu:8-23. */
int pie_hip_embed(const uint32_t* token_ids, const uint16_t* table_bf16, uint16_t* y_bf16,
                  int num_tokens, int hidden, int vocab, void* stream);

/* y = bf16( x * rsqrt(mean(x^2) + eps) * w ), fp32 inside.  hidden % 8 == 0.
 * Reference: rmsnorm_bf16_kernel, driver/cuda/src/kernels/rmsnorm.cu:14-54. */
int pie_hip_rmsnorm(const uint16_t* x_bf16, const uint16_t* weight_bf16, uint16_t* y_bf16,
                    int rows, int hidden, float eps, void* stream);

/* hidden = bf16(hidden + residual) (stored), norm_out = rmsnorm(hidden) of the rounded sum.
 * Reference: residual_add_rmsnorm_bf16_kernel, driver/cuda/src/kernels/rmsnorm.cu:56-98. */
int pie_hip_residual_rmsnorm(uint16_t* hidden_bf16, const uint16_t* residual_bf16,
                             const uint16_t* weight_bf16, uint16_t* norm_out_bf16, int rows,
                             int hidden, float eps, void* stream);

/* table[n, i] = cos(positions[n] * inv_freq[i]); table[n, i + d/2] = sin(same), i < d/2,
 * angle and sincos in fp32.  inv_freq[d/2] is a host table (theta^(-2i/d), optionally with
 * llama3 band scaling, driver/portable/src/model.cpp:1414-1448).
 * Reference: rope_standard_table_kernel, driver/cuda/src/kernels/rope.cu:35-53. */
int pie_hip_rope_table(const int32_t* positions, const float* inv_freq, float* table,
                       int num_tokens, int head_dim, void* stream);
/* The same with cos and sin multiplied by mscale (> 0): YaRN's attention factor
 * (rope_yarn_original_bf16_kernel, driver/cuda/src/kernels/rope.cu:509-548; the frequencies of
 * that scheme are a host-side inv_freq table like any other). */
int pie_hip_rope_table_scaled(const int32_t* positions, const float* inv_freq, float* table,
                              int num_tokens, int head_dim, float mscale, void* stream);

/*
 * Split a packed QKV row [N, (hq + 2*hk)*d], apply optional per-head RMSNorm (both norm
 * weights or neither) and RoPE to q and k, write q to q_out[N, hq, d], and write k (rotated)
 * and v (copied) into the KV pool [pages, page_size, hk, d] at physical slot
 * kv_slots[n] = page*page_size + offset (negative = token has no slot).  One bf16 rounding at
 * the store.  interleaved: PIE_HIP_ROPE_HALF (0) pairs (i, i+d/2), PIE_HIP_ROPE_ADJACENT (1) pairs
 * (2i, 2i+1), PIE_HIP_ROPE_HALF_PAIRED_ROWS (2): the q / k rows of the projection were re-ordered
 * at load so that elements (2i, 2i+1) of packed_qkv hold the half-split pair (i, i+d/2); they are
 * rotated as that pair and written to positions i and i+d/2 (V rows are as stored) — the output
 * of mode 0 over the original row order, bit for bit.
 * Reference: launch_qkv_decode_qk_norm_rope_write_kv_bf16,
 * driver/cuda/src/kernels/split_packed.hpp:34-57, split_packed.cu:62-178; slot arithmetic of
 * driver/portable/src/plan.hpp:36-45 is done by the caller.
 */
int pie_hip_qkv_rope_kvwrite(const uint16_t* packed_qkv, uint16_t* q_out, uint16_t* k_pages,
                             uint16_t* v_pages, const uint16_t* q_norm_weight,
                             const uint16_t* k_norm_weight, const float* rope_table,
                             const int64_t* kv_slots, int num_tokens, int num_q_heads,
                             int num_kv_heads, int head_dim, int interleaved, float eps,
                             void* stream);

/* y[n, i] = bf16( g/(1+exp(-g)) * u ), g = gate_up[n, i], u = gate_up[n, I + i].
 * Reference: swiglu_bf16_kernel, driver/cuda/src/kernels/swiglu.cu:9-22 (fused-row form
 * swiglu.hpp:82). */
int pie_hip_swiglu(const uint16_t* gate_up_bf16, uint16_t* y_bf16, int num_tokens,
                   int intermediate, void* stream);

/* out_idx[r] = argmax_i logits[r, i]; ties -> lowest index; NaN never wins.  vocab % 8 == 0.
 * Reference: argmax_bf16_kernel, driver/cuda/src/kernels/argmax.cu:36-80. */
int pie_hip_argmax(const uint16_t* logits_bf16, uint32_t* out_idx, int rows, int vocab,
                   void* stream);

/* pool page dst_pages[i] <- page src_pages[i] (device arrays), page_bytes each, in one pool.
 * Reference: Copy D2D handling, driver/portable/src/service/inproc_service.cpp:149-172. */
int pie_hip_copy_kv_pages(void* pool, const uint32_t* src_pages, const uint32_t* dst_pages,
                          int num_copies, size_t page_bytes, void* stream);

/* ---- load-time quantisers (bf16 weights -> storage formats) ---------------------- */

/* Per-output-channel int8: scale_inv[r] = absmax/127 (1 for a zero row),
 * q = clamp(rintf(w * 127/absmax), -128, 127), round half to even.
 * Reference: quantize_bf16_to_int8_per_channel, driver/cuda/src/kernels/quant_bf16_to_fp8.cu:273-333. */
int pie_hip_quant_int8_per_channel(const uint16_t* w_bf16, int8_t* q, float* scale_inv, int rows,
                                   int cols, void* stream);
/* Per-output-channel fp8 e4m3fn: scale_inv[r] = absmax/448, q = e4m3_satfinite(w * 448/absmax).
 * Reference: quant_per_channel_kernel, driver/cuda/src/kernels/quant_bf16_to_fp8.cu:181-226. */
int pie_hip_quant_fp8_per_channel(const uint16_t* w_bf16, uint8_t* q_e4m3, float* scale_inv,
                                  int rows, int cols, void* stream);
/* Symmetric group-wise int4 into the int4b8 layout: scale = bf16(absmax/7) per (row, group)
 * (1 for a zero group), nibble = clamp(rintf(w/scale), -8, 7) + 8.  The reference defines the
 * layout (driver/cuda/src/kernels/dequant_wna16.cu:11-38) but ships no quantiser for it. */
int pie_hip_quant_int4b8_group(const uint16_t* w_bf16, uint32_t* packed, uint16_t* scale_bf16,
                               int rows, int cols, int group_size, void* stream);

/* ---- layer stacks --------------------------------------------------------------- */
/*
 * Kernels of models whose layers are listed one by one (latent attention, gated delta rule,
 * squared-ReLU feed-forward, norms on the sublayers' outputs).  No counterpart in the reference.
 * dtype: the compute type, i.e. the storage of activations, of the latent cache and of the
 * convolution state (void pointers below).  Weights of products are bf16 in both types; norms,
 * angles, softmax, recurrences and the residual stream are fp32 in both.
 */
#define PIE_HIP_DT_BF16 0
#define PIE_HIP_DT_F32 1

/* x[n, :] = table[token_ids[n], :] (ids >= vocab read row 0) in fp32 and, as x_act, in the compute
 * type; rows of ld values, columns from the width on are zero. */
int pie_hip_embed_stream(int dtype, const uint32_t* token_ids, const uint16_t* table_bf16, float* x,
                         void* x_act, int num_tokens, int width, int ld, int vocab, void* stream);
/* x += y / sqrt(mean(y^2) + eps) * weight; x_act = the new x in the compute type. */
int pie_hip_norm_add(int dtype, const void* y, const float* weight, float* x, void* x_act, int rows, int width,
                     int ldy, int ld, float eps, void* stream);
/* out[s, :] = x[rows[s], :] / sqrt(mean(x^2) + eps) * weight in the compute type (zeros from the
 * width to ld). */
int pie_hip_norm_rows(int dtype, const float* x, const uint32_t* rows, const float* weight, void* out,
                      int num_out, int width, int ld, int num_rows, float eps, void* stream);
/* logits[s, v] = cap * tanh(y[s, v] * scale / cap) (cap 0: y * scale) in fp32, and tokens[s], the
 * index of the largest (lowest among equals, NaN never wins). */
int pie_hip_logits_finish(int dtype, const void* y, float* logits, uint32_t* tokens, int rows, int vocab,
                          int ldy, float scale, float cap, void* stream);
/* table[n, i] = cos(a) * mscale, table[n, dims/2 + i] = sin(a) * mscale with a = positions[n] *
 * freq[i]; angles are formed and reduced in double. */
int pie_hip_rotary_table(const int32_t* positions, const double* freq, float* table, int num_tokens, int dims,
                         float mscale, void* stream);
/* y[M, N] = act[M, K] . W[N, K]^T in fp32 over bf16 weights; epilogue PIE_HIP_EPI_NONE / _RELU2. */
int pie_hip_linear_f32(const float* act, const uint16_t* w_bf16, float* y, int M, int N, int K, int epilogue,
                       void* stream);

/*
 * Latent attention.  A cache row is [kvp latent | rotated key part] (ld_row values, zero padded);
 * the pool is [pages * page_size, ld_row], one per layer, kv_slots / page lists as for the K / V
 * pools.
 * pie_hip_latent_prep: fused[n] = [query latent q_rank | .. | kv_off: latent kv_rank, rot_dim key
 *   values]; cq[n] = the query latent normed (compact rows of ld_cq, zero padded); the token's
 *   cache row = the normed latent and the key values rotated in adjacent pairs (first rot_dims of
 *   them, table of pie_hip_rotary_table).  kv_norm NULL: only the query latent (fused holds nothing else).
 * pie_hip_head_linear: y[n, h, c] = sum_k W[h, c, k] act[n, h, k] (heads act_stride / y_stride
 *   apart in rows of ld_act / ld_y; C % 16 == 0, K % 32 == 0).  With rotp > 0 also
 *   y[n, h, C + i] = the rotated act[n, h, rot_off + i], i < rot_dim, zeros to rotp.  With gate,
 *   y[n, h, c] is multiplied by the logistic function of gate[n, h * gate_cols + c % gate_cols] (rows of
 *   ld_gate; gate_cols C: one per value, 1: one per head).
 * pie_hip_latent_attn_rows_plain: o[n, h, :] = softmax_j(q[n, h, :] . row_j * scale) . row_j[:kvp]
 *   over the first row_kv_len[n] keys; q [rows, heads, ld_row], o [rows, heads, kvp].  Any sizes
 *   (kvp <= 2048).  sinks [heads] fp32 (NULL: none), in all forms of the attention: exp(sinks[h]) joins head
 *   h's sum of exponentials.
 */
int pie_hip_latent_prep(int dtype, const void* fused, const float* q_norm, const float* kv_norm,
                        const float* rope_table, const int64_t* kv_slots, void* cq, void* pool, int num_tokens,
                        int ld_fused, int kv_off, int q_rank, int ld_cq, int kv_rank, int kvp, int rot_dim,
                        int rot_dims, int ld_row, float eps, void* stream);
int pie_hip_head_linear(int dtype, const void* act, const uint16_t* w_bf16, void* y, const float* rope_table,
                        int M, int heads, int C, int K, int ld_act, int act_stride, int ld_y, int y_stride,
                        int rot_off, int rot_dim, int rot_dims, int rotp, const void* gate, int ld_gate,
                        int gate_cols, void* stream);
int pie_hip_latent_attn_rows_plain(int dtype, const void* q, const void* pool, void* o,
                                   const uint32_t* kv_page_indices, const uint32_t* row_page_begin,
                                   const int32_t* row_kv_len, int num_rows, int heads, int kvp, int ld_row,
                                   int page_size, float scale, const float* sinks, void* stream);

/* The same function on the matrix cores over bf16 pools, rows [row0, row0 + num_rows): weights
 * enter the second product as hi + lo bf16 pairs.  rotp in {0, 32, 64}, kvp in {64, 128, 192, 256, 384,
 * 512} (pie_hip_latent_attn_rows_supported), page_size % 16 == 0.  max_tokens_per_req: the most
 * rows a request brings (1: a decode batch; more: row_req / qo_indptr must cover the rows, whole
 * requests only).  workspace: pie_hip_latent_attn_rows_workspace_bytes. */
int pie_hip_latent_attn_rows_supported(int kvp, int rotp);
size_t pie_hip_latent_attn_rows_workspace_bytes(int num_rows, int heads, int kvp, int max_kv_len,
                                                int max_tokens_per_req);
int pie_hip_latent_attn_rows(const uint16_t* q, const uint16_t* pool, uint16_t* o, const uint32_t* kv_page_indices,
                             const uint32_t* row_page_begin, const int32_t* row_kv_len, const int32_t* row_req,
                             const int32_t* qo_indptr, int row0, int num_rows, int heads, int kvp, int rotp,
                             int page_size, float scale, const float* sinks, int max_kv_len,
                             int max_tokens_per_req, void* workspace, size_t workspace_bytes, void* stream);
/* Long portions: keys and values projected out of the latents, then ordinary causal attention.
 * pie_hip_latent_gather: the first num_keys cache rows of a page list as compact rows, lat [num_keys,
 *   kvp] and rot [num_keys, rotp].
 * pie_hip_latent_attn_prefill: rows [row0, row0 + num_rows) of one request, q [rows, heads, dimp +
 *   rotp] (the rotated part not yet rotated: rope_table rows as for pie_hip_latent_prep), kv
 *   [num_keys, heads, dimp + vdp] the projected keys and values, rot as gathered; row n sees its
 *   first row_kv_len[n] keys; o [rows, ld_o], heads vdp apart, times the logistic function of
 *   gate[n, h * gate_cols + c % gate_cols] (rows of ld_gate, gate_cols vdp or 1; NULL: none).  rot may be
 *   NULL with rotp 0.  (dimp + rotp) / 32 in 1..6, vdp / 32 in 1..4
 *   (pie_hip_latent_attn_prefill_supported). */
int pie_hip_latent_gather(const uint16_t* pool, const uint32_t* pages, uint16_t* lat, uint16_t* rot, int num_keys,
                          int kvp, int rotp, int page_size, void* stream);
int pie_hip_latent_attn_prefill_supported(int dimp, int rotp, int vdp);
int pie_hip_latent_attn_prefill(const uint16_t* q, const uint16_t* kv, const uint16_t* rot, uint16_t* o,
                                const float* rope_table, const int32_t* row_kv_len, int row0, int num_rows,
                                int num_keys, int heads, int dimp, int rotp, int rot_dims, int vdp, int ld_o,
                                float scale, const float* sinks, const uint16_t* gate, int ld_gate,
                                int gate_cols, void* stream);

/*
 * Gated delta rule with a decay per head and key channel.  row_req [N]: request of each row;
 * qo_indptr [R + 1]: rows of each request; rs_slot [R]: its slot of the state pool (rs_base + slot *
 * rs_stride bytes); rs_fresh [R]: 1 = starts from zero.  The fp32 state [heads, dim, vdim] sits at
 * state_offset of the slot, the last taps - 1 convolution inputs [taps - 1, channels] (compute type,
 * channels = q | k | v) at conv_offset.
 * pie_hip_delta_prep: fused[n] = [q | k | v | step sizes (heads) | ..].  q, k: causal convolution
 *   (conv_w [channels, taps], the last column is the current token's), silu, unit vector
 *   x / sqrt(sum x^2 + 1e-6) per head, q also times dim^-1/2; v: convolution, silu; beta =
 *   sigmoid(step size).  dim <= 512.
 * pie_hip_delta_conv_state: the last taps - 1 convolution inputs of every request (after prep).
 * pie_hip_delta_lowrank: fused[n] also holds the low-rank inputs a1 (decay_off, decay_rank) and g1
 *   (gate_off, gate_rank); log2_decay = rate[head] softplus(w_decay a1 + dt_bias) with
 *   rate = -exp(A_log) log2(e), [N, heads * dim] fp32; gate = w_gate g1, [N, ld_gate] compute type.  Weights [.., ld_a1], [..,
 *   ld_g1], zero past the ranks.
 * pie_hip_delta_scan: per token S <- g S, u = beta (v - S^T k), S <- S + k u^T, o = S^T q with g =
 *   2^log2_decay; head h uses q / k head h / (heads / kv_heads).  Reads and writes the state.
 *   dim <= 256.
 * pie_hip_delta_chunked: the same recurrence sixteen tokens at a time on the fp32 matrix
 *   instructions.  chunks [num_chunks][2] = (first row, rows <= 16), a request's in order;
 *   req_chunks [R + 1].  dim <= 256; workspace pie_hip_delta_chunked_workspace_bytes.
 * pie_hip_delta_out: y = o / sqrt(mean(o^2) + eps) * norm_w * sigmoid(gate) per head.
 * pie_hip_delta_step: prep, scan and out for one token per request (row r = request r) in one launch;
 *   write_conv (heads == kv_heads only) moves the convolution's state on too.  vdim a multiple of 4,
 *   dim and vdim <= 256 (pie_hip_delta_step_supported).
 */
int pie_hip_delta_prep(int dtype, const void* fused, const float* conv_w, const void* rs_base, size_t rs_stride,
                       size_t conv_offset, const int32_t* row_req, const int32_t* qo_indptr,
                       const int32_t* rs_slot, const int32_t* rs_fresh, float* q, float* k, float* v, float* beta,
                       int num_tokens, int ld, int heads, int kv_heads, int dim, int vdim, int taps, void* stream);
int pie_hip_delta_conv_state(int dtype, const void* fused, void* rs_base, size_t rs_stride, size_t conv_offset,
                             const int32_t* qo_indptr, const int32_t* rs_slot, const int32_t* rs_fresh,
                             int num_requests, int ld, int channels, int taps, void* stream);
int pie_hip_delta_lowrank(int dtype, const void* fused, const uint16_t* w_decay, const uint16_t* w_gate,
                          const float* rate, const float* dt_bias, float* log2_decay, void* gate, int num_tokens,
                          int ld, int decay_off, int decay_rank, int ld_a1, int gate_off, int gate_rank, int ld_g1,
                          int heads, int dim, int vdim, int ld_gate, void* stream);
int pie_hip_delta_scan(const float* q, const float* k, const float* v, const float* log2_decay, const float* beta,
                       float* o, void* rs_base, size_t rs_stride, size_t state_offset, const int32_t* qo_indptr,
                       const int32_t* rs_slot, const int32_t* rs_fresh, int num_requests, int heads, int kv_heads,
                       int dim, int vdim, void* stream);
size_t pie_hip_delta_chunked_workspace_bytes(int num_chunks, int heads, int dim);
int pie_hip_delta_chunked(const float* q, const float* k, const float* v, const float* log2_decay, const float* beta,
                          float* o, void* rs_base, size_t rs_stride, size_t state_offset, const int32_t* chunks,
                          const int32_t* req_chunks, const int32_t* qo_indptr, const int32_t* rs_slot,
                          const int32_t* rs_fresh, int num_chunks, int num_requests, int heads, int kv_heads, int dim, int vdim, void* workspace,
                          size_t workspace_bytes, void* stream);
int pie_hip_delta_out(int dtype, const float* o, const void* gate, const float* norm_w, void* y, int num_tokens,
                      int ld_gate, int ld_y, int heads, int vdim, float eps, void* stream);
int pie_hip_delta_step_supported(int dim, int vdim);
int pie_hip_delta_step(int dtype, const void* fused, const float* conv_w, const float* log2_decay, const void* gate,
                       const float* norm_w, void* y, void* rs_base, size_t rs_stride, size_t state_offset,
                       size_t conv_offset, const int32_t* rs_slot, const int32_t* rs_fresh, int num_requests, int ld,
                       int ld_gate, int ld_y, int heads, int kv_heads, int dim, int vdim, int taps, int write_conv,
                       float eps, void* stream);

/* One step of the residual stream of layers with norms ahead of and after their sublayers:
 *   x[n] = (read_x ? x[n] : 0) + y[n] / sqrt(mean(y[n]^2) + eps) * post_weight + table[token_ids[n]] + add
 *   x_act[n] = x[n] / sqrt(mean(x[n]^2) + eps) * next_weight        (compute type)
 * y with post_weight, token_ids with table_bf16, and add [width] may each be NULL (left out);
 * next_weight NULL: x_act = x.  ids >= vocab read row 0.  Columns from the width to ld are not touched. */
int pie_hip_residual_norm(int dtype, const void* y, const float* post_weight, float* x, int read_x,
                          const uint32_t* token_ids, const uint16_t* table_bf16, int vocab, const float* add,
                          const float* next_weight, void* x_act, int rows, int width, int ldy, int ld, float eps,
                          void* stream);
/* What a mixture of experts leaves per token: its routes' rows y (compute type, rows of ld), the row pos[t, k]
 * of each route and its weight [t, k]. */
typedef struct {
    const void* y;
    const int32_t* pos;
    const float* weight;
    int top_k, ld;
} PieHipRoutes;
/* One step of the residual stream of layers whose sublayers read one norm and join the stream together:
 *   x[n] = (read_x ? x[n] : 0) + y[n] + y2[n] + add + sum_k weight[n, k] routes.y[pos[n, k]] + table[token_ids[n]] *
 *          table_scale
 *   x_act[n] = x[n] / sqrt(mean(x[n]^2) + eps) * next_weight        (compute type)
 * y (rows of ldy), y2 (rows of ldy2), add [width], routes and token_ids with table_bf16 may each be NULL (left
 * out); next_weight NULL: x_act = x.  ids >= vocab read row 0.  Columns from the width to ld are not touched. */
int pie_hip_residual_join(int dtype, const void* y, int ldy, const void* y2, int ldy2, const float* add,
                          const PieHipRoutes* routes, float* x, int read_x, const uint32_t* token_ids,
                          const uint16_t* table_bf16, int vocab, float table_scale, const float* next_weight,
                          void* x_act, int rows, int width, int ld, float eps, void* stream);
/* The fp32 forms of a mixture's products and of the gated rule:
 * pie_hip_moe_grouped_linear_f32: rows expert_offsets[e] .. expert_offsets[e + 1] of y [routes, N] are
 *   act[route_act_rows[r]] (or act[r]) . W_e^T, W_e bf16 [N, K] at w + e * N * K; no expert has more than
 *   max_rows; epilogue as for pie_hip_linear_f32.
 * pie_hip_glu_f32: y[m, i] = the rule of PieHipGlu on columns (2i, 2i + 1) of x [M, 2 n]. */
int pie_hip_moe_grouped_linear_f32(const float* act, const int32_t* route_act_rows, const int32_t* expert_offsets,
                                   int num_experts, int max_rows, const uint16_t* w_bf16, float* y, int N, int K,
                                   int epilogue, void* stream);
int pie_hip_glu_f32(const float* x, const PieHipGlu* glu, float* y, int M, int n, void* stream);
/* y[M, N] fp32 = act[M, K] . W[N, K]^T over bf16 weights (fp32 sums, not rounded): the few columns that
 * drive a recurrence.  K % 32 == 0, N % 16 == 0. */
int pie_hip_linear_f32out(int dtype, const void* act, const uint16_t* w_bf16, float* y, int M, int N, int K,
                          void* stream);

/*
 * Grouped-query attention with an optional sliding window (a row sees its last `window` keys, itself
 * included; 0: all), an optional sink (`sink` is added to the sum of exponentials; 0: none), and any
 * head size.  Cache rows: [kv_heads][key dimp | value dimp], dim padded with zeros to dimp; the pool is
 * [pages * page_size, row], one per layer run.
 * pie_hip_group_attn_prep: fused[n] holds q (heads * dim from q_off), k and v (kv_heads * dim from k_off /
 *   v_off; v_off < 0: the values are the keys as projected).  Biases (or NULL) are added, q and k are
 *   normed per head (weights [dim], or NULL) and rotated over their first rot_dims entries, entry i
 *   with entry i + rot_dims / 2 (table of pie_hip_rotary_table); q goes to q_out [N, heads, dimp].
 * pie_hip_group_attn_rows: one query row per block row; rows NULL: rows 0 .. num_rows - 1, else the
 *   listed ones.  o[row, h * dimp ..] * out_scale, rows of ld_o, in all three forms also times the
 *   logistic function of gate[row, h * dimp ..] (rows of ld_gate; NULL: none).  bf16; dimp / 32 in {1, 2, 3, 4, 6, 8};
 *   page_size % 16 == 0.  Workspace pie_hip_group_attn_rows_workspace_bytes.
 * pie_hip_group_attn_tiles: tiles [num_tiles][2] = (first row, rows) of consecutive rows of one request,
 *   at most pie_hip_group_attn_tile_rows(heads, kv_heads, half) of them; half tiles only for dimp > 128.
 * pie_hip_group_attn_plain: any size and compute type, dimp <= 1024.
 * pie_hip_group_attn_prep_joint: as pie_hip_group_attn_prep without biases, with one norm over a row's whole
 *   query projection and one over its whole key projection (weights [heads * dim] and [kv_heads * dim], or
 *   NULL), values of their own size vdim <= dimp, and either pairing of the rotated entries
 *   (PIE_HIP_ROPE_HALF or PIE_HIP_ROPE_ADJACENT).
 */
int pie_hip_group_attn_prep(int dtype, const void* fused, int q_off, int k_off, int v_off, const float* q_bias,
                            const float* k_bias, const float* q_norm, const float* k_norm, const float* rope_table,
                            int rot_dims, const int64_t* kv_slots, void* q_out, void* pool, int num_tokens,
                            int ld_fused, int heads, int kv_heads, int dim, int dimp, float eps, void* stream);
int pie_hip_group_attn_prep_joint(int dtype, const void* fused, int q_off, int k_off, int v_off, const float* q_norm,
                                  const float* k_norm, const float* rope_table, int rot_dims, int pairing,
                                  const int64_t* kv_slots, void* q_out, void* pool, int num_tokens, int ld_fused,
                                  int heads, int kv_heads, int dim, int vdim, int dimp, float eps, void* stream);
int pie_hip_group_attn_supported(int dimp);
size_t pie_hip_group_attn_rows_workspace_bytes(int num_rows, int heads, int kv_heads, int dimp, int max_kv_len, int window);
int pie_hip_group_attn_rows(const uint16_t* q, const uint16_t* pool, uint16_t* o, const uint32_t* kv_page_indices,
                            const uint32_t* row_page_begin, const int32_t* row_kv_len, const int32_t* rows,
                            int num_rows, int heads, int kv_heads, int dimp, int ld_o, int page_size, float scale,
                            int window, float sink, float out_scale, const uint16_t* gate, int ld_gate,
                            int max_kv_len, void* workspace,
                            size_t workspace_bytes, void* stream);
int pie_hip_group_attn_tile_rows(int heads, int kv_heads, int half);
int pie_hip_group_attn_tiles(const uint16_t* q, const uint16_t* pool, uint16_t* o, const uint32_t* kv_page_indices,
                             const uint32_t* row_page_begin, const int32_t* row_kv_len, const int32_t* tiles,
                             int num_tiles, int half, int heads, int kv_heads, int dimp, int ld_o, int page_size,
                             float scale, int window, float sink, float out_scale, const uint16_t* gate,
                             int ld_gate, void* stream);
int pie_hip_group_attn_plain(int dtype, const void* q, const void* pool, void* o, const uint32_t* kv_page_indices,
                             const uint32_t* row_page_begin, const int32_t* row_kv_len, int num_rows, int heads,
                             int kv_heads, int dimp, int ld_o, int page_size, float scale, int window, float sink,
                             float out_scale, const void* gate, int ld_gate, void* stream);

/*
 * Memories with one decay per head and token: S_t = d_t S_(t-1) + w_t k_t v_t^T (S [dim, vdim] fp32),
 * o_t = S_t^T q_t.  Query and key heads may be shared: head h uses head h / (heads / kv_heads).
 * The rule gives d_t and w_t (gates: fp32 rows of ld_gates values per token):
 *   FIXED      d = 2^decay[head], w = k_scale                                         (retention)
 *   EXP_GATES  i = cap tanh((gates[h] + gate_bias[h]) / cap), f = log sigmoid(cap tanh((gates[heads + h] +
 *              gate_bias[heads + h]) / cap)), m_t = max(f + m_(t-1), i), d = exp(f + m_(t-1) - m_t), w =
 *              exp(i - m_t); a vector n with v = 1 beside S; o is divided by max(|n . q|, exp(-m_t)) +
 *              1e-6 in pie_hip_decay_out                                                       (mLSTM)
 *   STEP       dt = softplus(gates[h] + gate_bias[h]), d = 2^(decay[h] dt), w = dt            (Mamba-2)
 * o is also multiplied by q_scale.  A request's state: S [heads, dim, vdim], then (EXP_GATES) n [heads,
 * dim] and m [heads] in units of log 2, at state_offset of its slot; the last taps - 1 inputs of a
 * convolution ([taps - 1, channels], compute type) at conv_offset.
 */
#define PIE_HIP_DECAY_FIXED 0
#define PIE_HIP_DECAY_EXP_GATES 1
#define PIE_HIP_DECAY_STEP 2
typedef struct {
    int kind, heads, kv_heads, dim, vdim;
    float q_scale, k_scale, gate_cap;
    const float* decay;       /* [heads]: FIXED log2 of the decay; STEP -exp(A_log) log2(e) */
    const float* gate_bias;   /* EXP_GATES [2 heads]; STEP [heads] */
} PieHipDecayRule;
/* Which rows of the batch a request owns and where its state lives. */
typedef struct {
    const int32_t* row_req;     /* [num_tokens] */
    const int32_t* qo_indptr;   /* [num_requests + 1] */
    const int32_t* rs_slot;     /* [num_requests] */
    const int32_t* rs_fresh;    /* [num_requests] 1: starts from zero */
    void* rs_base;
    size_t rs_stride, state_offset, conv_offset;   /* bytes */
    int num_tokens, num_requests;
} PieHipStateRows;
/* out[n, c] = silu(bias[c] + sum_j conv_w[c, j] * input_(n - (taps - 1) + j)[c]) for the first `channels`
 * columns of fused (earlier inputs from the state, zeros before the start); rows of ld_out.
 * move_state (one row per request only): the state also moves on by that row; elsewhere
 * pie_hip_delta_conv_state does it afterwards. */
int pie_hip_conv_silu(int dtype, const void* fused, const float* conv_w, const float* conv_bias,
                      const PieHipStateRows* rows, void* out, int ld, int channels, int taps, int ld_out,
                      int move_state, void* stream);
/* Token by token, any compute type: q, k, v rows of ld values.  o [N, heads * vdim] fp32; den [N, heads, 2]
 * (EXP_GATES: n . q and m_t).  dim <= 512. */
int pie_hip_decay_scan(int dtype, const PieHipDecayRule* rule, const PieHipStateRows* rows, const void* q,
                       const void* k, const void* v, int ld, const float* gates, int ld_gates, float* o, float* den,
                       void* stream);
/* 64 tokens at a time on the matrix cores (bf16).  chunks [num_chunks][2] = (first row, rows <= 64), a
 * request's in order; req_chunks [num_requests + 1].  dim <= 512. */
size_t pie_hip_decay_chunked_workspace_bytes(const PieHipDecayRule* rule, int num_chunks);
int pie_hip_decay_chunked(const PieHipDecayRule* rule, const PieHipStateRows* rows, const uint16_t* q,
                          const uint16_t* k, const uint16_t* v, int ld, const float* gates, int ld_gates, float* o,
                          float* den, const int32_t* chunks, const int32_t* req_chunks, int num_chunks,
                          void* workspace, size_t workspace_bytes, void* stream);
/* y[n, h * vdim + c] = out_scale * o' / sqrt(mean(o'^2) + eps) * norm_w[h * vdim + c] * act(gate[n, h * vdim + c]),
 * o' = o, divided for EXP_GATES as above (and m_t of a request's last row goes to its state).  norm_w may
 * be NULL; gate_act 0: sigmoid, 1: silu. */
int pie_hip_decay_out(int dtype, const PieHipDecayRule* rule, const PieHipStateRows* rows, const float* o,
                      const float* den, const void* gate, int ld_gate, int gate_act, const float* norm_w, void* y,
                      int ld_y, float out_scale, float eps, void* stream);
/* One token per request (row r = request r), one launch: the state is read and written once.  conv_w not
 * NULL: q, k, v are columns q_off, k_off, v_off of `fused` ahead of the convolution (conv_w [channels, taps] indexed
 * by the same columns; the state is read, not moved on).  skip not NULL: skip[head] * v is added to o.  y not NULL: with
 * pie_hip_decay_out's norm and gate fused (one block per head then), else o and den.
 * vdim % 4 == 0, dim <= 512, vdim <= 1024 (pie_hip_decay_step_supported). */
int pie_hip_decay_step_supported(int dim, int vdim);
int pie_hip_decay_step_fuses(const PieHipDecayRule* rule, int num_requests);
int pie_hip_decay_step(int dtype, const PieHipDecayRule* rule, const PieHipStateRows* rows, const void* fused,
                       int q_off, int k_off, int v_off, int ld, const float* gates, int ld_gates, const float* conv_w,
                       const float* conv_bias, int channels, int taps, const float* skip, float* o, float* den,
                       const void* gate, int ld_gate, int gate_act, const float* norm_w, void* y, int ld_y,
                       float out_scale, float eps, void* stream);
/* y = g / sqrt(mean over its part (g^2) + eps) * norm_w, g = (o + skip[head] * x) * silu(z), the heads * vdim
 * values of a row in `parts` equal parts; x NULL: o as it is.  conv_w taps > 1 and conv_fused not NULL (one row
 * per request): the convolution's state also moves on by the row's inputs. */
int pie_hip_gated_part_norm(int dtype, const float* o, const void* x, int ld_x, const float* skip, const void* z,
                            int ld_z, const float* norm_w, void* y, int ld_y, int heads, int vdim, int parts,
                            const PieHipStateRows* rows, const void* conv_fused, int ld_fused, int channels, int taps,
                            float eps, void* stream);

/*
 * Layers whose sublayers' outputs pass a logistic gate and whose sublayers read a short convolution of the normed
 * stream: h = norm(x), the sublayer reads h + conv(h), x += sublayer * sigmoid(gate), the gate a product of h.
 * pie_hip_gated_join: x[n] += (y[n] or a mixture's routes, see PieHipRoutes) * sigmoid(gate[n] + gate_bias) (neither y
 *   nor routes: x as it is; with `start` x is set to an embedding, see PieHipEmbedding); h[n] = x[n] / sqrt(mean(x[n]^2) + eps) * next_weight in the compute type (next_weight
 *   NULL: x only).  With conv_w (one row per request, taps <= 4) also recent[n] = h[n] + the convolution, whose
 *   state moves on by the row.  Rows of ld; columns from the width on are not touched.
 * pie_hip_recent_rows: recent[n, c] = h[n, c] + sum_j conv_w[j, c] h_(n - (taps - 1) + j)[c], earlier rows from the
 *   request's state, zeros before its start; pie_hip_delta_conv_state (channels = width) moves the state on
 *   afterwards.  conv_w [taps, width] bf16; the state is [taps - 1, width] in the compute type at conv_offset.
 */
/* x[n] = e / sqrt(mean(e^2) + eps) * norm_weight, e = table[token_ids[n]] * scale + pair_table[pair_rows[n]] (pair_table
 * NULL: left out; ids >= vocab read row 0 of table). */
typedef struct {
    const uint32_t* token_ids;
    const int32_t* pair_rows;
    const uint16_t *table, *pair_table;
    const float* norm_weight;
    int vocab;
    float scale;
} PieHipEmbedding;
int pie_hip_gated_join(int dtype, const void* y, int ldy, const PieHipRoutes* routes, const void* gate, int ld_gate,
                       const float* gate_bias, const PieHipEmbedding* start, float* x, const float* next_weight,
                       void* h, void* recent, const uint16_t* conv_w, int taps, const PieHipStateRows* state, int rows, int width, int ld,
                       float eps, void* stream);
int pie_hip_recent_rows(int dtype, const void* h, const uint16_t* conv_w, int taps, const PieHipStateRows* state, void* recent,
                        int width, int ld, void* stream);
/* The sorted layout of pie_hip_moe_route_groups for a router of logistic scores s = sigmoid(logit): a token uses the
 * top_k experts with the largest s + correction (lowest index among equals), weighted by their s.  `shared` experts
 * that every token uses come ahead of them, as experts 0 .. shared - 1, weighted by sigmoid(logits[t, num_experts]);
 * the routed ones are numbered from `shared` on.  topk_idx and topk_weight [T, shared + top_k],
 * expert_offsets [shared + num_experts + 1]. */
int pie_hip_moe_route_corrected(const float* router_logits, int ld_logits, const float* correction, int32_t* topk_idx,
                                float* topk_weight, int32_t* expert_offsets, int32_t* route_token, int32_t* route_pos,
                                int num_tokens, int num_experts, int top_k, int shared, void* stream);

/* pie_hip_sample_gather_logits over fp32 logits. */
int pie_hip_sample_gather_logits_f32(const float* logits, const int32_t* rows, float* out_f32,
                                     const uint32_t* mask_bounds, const int32_t* mask_bounds_indptr,
                                     int num_slots, int vocab, void* stream);

#ifdef __cplusplus
}
#endif
#endif /* PIE_HIP_KERNELS_H */
