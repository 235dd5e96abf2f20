/*
 * tunix_hip.h -- C ABI of libtunix_hip.so: hand-written gfx950 (MI355X) kernels for the
 * quantized rollout-decode path of google/tunix (Sampler decode step on int4/NF4 QLoRA
 * models + per-token logps).
 *
 * Conventions (all entry points):
 *   - extern "C"; `stream` is a hipStream_t passed as void* (NULL = the null stream);
 *   - every pointer is a DEVICE pointer unless its name starts with `h_`;
 *   - no allocation, no synchronisation, no host callback inside; outputs are caller-allocated;
 *   - in-place updates (KV cache, token buffer) use the same pointer for input and output;
 *   - return 0 on success, a negative TNX_E* code otherwise; tnx_last_error() returns the
 *     calling thread's last message;
 *   - bf16 values are raw uint16_t bit patterns; all matrices are row-major;
 *   - scalars that change from one decode step to the next (step index, positions) are read
 *     from device memory so that a captured HIP graph of one step can be replayed unchanged.
 *
 * Each declaration cites the reference code (paths relative to the google/tunix tree) whose
 * arithmetic the entry point replaces.
 */
#ifndef TUNIX_HIP_H_
#define TUNIX_HIP_H_

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

#define TNX_OK 0
#define TNX_EINVAL (-22)  /* bad shape / alignment / enum                         */
#define TNX_ELAUNCH (-5)  /* hipGetLastError() != hipSuccess after a kernel launch */
#define TNX_ENOSYS (-38)  /* combination not built                                 */

/* Weight code books. INT4: code u in [0,15] means the integer u-8. NF4: the 16 QLoRA levels. */
#define TNX_Q_INT4 0
#define TNX_Q_NF4 1

/* RMSNorm dtype flows (tunix/models/llama3/model.py:290-297, qwen3/model.py:450-456,
 * gemma3/model.py:940-950). */
#define TNX_NORM_LLAMA 0
#define TNX_NORM_QWEN3 1
#define TNX_NORM_GEMMA3 2

/* RoPE dtype flows (llama3/model.py:249-270 fp32 sin/cos; qwen3/model.py:404-425 sin/cos
 * rounded to bf16 first; gemma3/model.py:402-430 fp32 with base frequency + scale factor). */
#define TNX_ROPE_LLAMA 0
#define TNX_ROPE_QWEN3 1
#define TNX_ROPE_GEMMA3 2

/* Epilogues of tnx_qlinear_lora. */
#define TNX_EPI_STORE 0     /* y = bf16(acc)                                               */
#define TNX_EPI_RESIDUAL 1  /* y = bf16(bf16(acc) + residual)      (llama3/model.py:560-563) */
#define TNX_EPI_SILU_MUL 2  /* y = bf16(bf16(silu(bf16 g)) * bf16 u) (llama3/model.py:493)    */
#define TNX_EPI_GELU_MUL 3  /* y = bf16(bf16(gelu_tanh(bf16 g)) * bf16 u) (gemma3/model.py:785-797) */
#define TNX_EPI_F32 4       /* y(fp32) = acc, no rounding                                   */
#define TNX_EPI_RELU2 5     /* y = max(acc, 0)^2 (tnx_dense_linear alone)                   */

const char* tnx_last_error(void);
/* Library / ABI version: (major << 16) | minor, the value tnx_version() returns.
 * Rule: the MAJOR number changes whenever an existing entry point changes its argument list or
 * meaning, or a descriptor struct changes its layout (a field added, removed, moved or retyped):
 * a caller built against another major number must not call the library.  The MINOR number counts
 * additions that leave every existing entry point and struct exactly as they were (new entry
 * points, new enum values); a caller built against minor m runs on any minor >= m of the same
 * major.  A caller checks tnx_version() >> 16 == TNX_ABI_VERSION_MAJOR and
 * (tnx_version() & 0xffff) >= TNX_ABI_VERSION_MINOR before its first call.
 * History: 1.0 first ABI; 1.1 added tnx_rmsnorm_moe_combine (and, against this rule, an argument
 * of tnx_quantize_pack and a field of tnx_lmhead_desc); 2.0 states the rule, keeps those changes,
 * adds tnx_attn_desc.segment_ids, reads top_k == V in tnx_sample_topk as a real top-k, and moves
 * the measurement probe tnx_stream_read out of the library; 3.0 adds tnx_qw_expand /
 * tnx_qw_expanded_bytes, tnx_dense_expand and the w_expanded field of tnx_qlinear_desc and
 * tnx_lmhead_desc; 3.1 adds tnx_sample_topk_head / tnx_sample_topk_head_ok; 3.2 adds the entry
 * points of decoders with dense weights (tnx_dense_linear to tnx_logits_stats); 4.0 adds batches and experts
 * to tnx_dense_desc, parts, routed rows and the token shift to tnx_residual_norm_desc, the gate in front
 * to tnx_gated_norm_desc, out_head to tnx_sink_attn_desc, and tnx_silu_mul, tnx_route_softmax,
 * tnx_short_conv, tnx_ring_write, tnx_ssd, tnx_latent_* and tnx_gate_mul; 5.0 adds softcap to tnx_lmhead_desc,
 * a scale to tnx_embed_rows, a first column to tnx_ring_write, parts behind the norm of tnx_gated_norm, and
 * tnx_parallel_step, tnx_conv_kvwrite, tnx_mixed_attn, tnx_memory and tnx_soft_cap; 6.0 adds learned positions to
 * tnx_embed_rows, centred norms, a factor, an extra row and the depth average to tnx_residual_norm_desc, slopes and
 * chunks to tnx_sink_attn_desc, an ungated form and shared weights to tnx_gated_norm_desc, TNX_EPI_RELU2, and
 * tnx_rownorm_kvwrite, tnx_gated_state, tnx_poly_norm and tnx_route_scores. */
#define TNX_ABI_VERSION_MAJOR 6
#define TNX_ABI_VERSION_MINOR 0
#define TNX_ABI_VERSION ((TNX_ABI_VERSION_MAJOR << 16) | TNX_ABI_VERSION_MINOR)
int tnx_version(void);

/* ---------------------------------------------------------------------------------------
 * Packed weight format ("QW"), defined by this library (qwix's QArray layout is third-party
 * and not part of the reference tree; tunix only passes weight_qtype / tile_size through at
 * tunix/cli/utils/model.py:31-77).
 *
 * A linear y[M,N] = x[M,K] . W[K,N] is quantized in groups of `group` consecutive K indices
 * per output column: scale[g,n] = bf16(absmax / 7) (INT4) or bf16(absmax) (NF4); the code of
 * an element is the nearest code-book entry of w / f32(scale) (round-half-even for INT4,
 * clamped to [-8,7]; nearest level, ties to the lower code, for NF4).  The value a kernel
 * uses is the weight dequantised to bf16,  w^[k,n] = bf16( bf16(level(code)) * scale[g(k),n] ),
 * multiplied into bf16 activations with fp32 accumulation:  y[m,n] = sum_k x[m,k] * w^[k,n].
 *
 * Storage: N is padded to a multiple of 16 and K to a multiple of 128. Codes are tiled as
 * [N/16][K/128][64 lanes][4 dwords]; lane l of a tile owns column n = 16*nt + l%16; its dword
 * j holds the 8 codes of k = 128*kt + 32*j + 8*(l/16) + i, i = 0..7, code i in bits 4i..4i+3.
 * Scales are tiled as [N/16][K/128][16][S] bf16 with S = max(2, 128/group) slots per k-tile
 * and column, slot s holding the scale of k = 128*kt + s*(128/S) .. (a group wider than a slot
 * repeats its scale), so that a lane reads its scales as one aligned 4- or 8-byte word.
 * tnx_qw_sizes() gives the byte sizes; tnx_quantize_pack() produces both arrays on device.
 * ------------------------------------------------------------------------------------- */
int tnx_qw_sizes(int64_t K, int64_t N, int group, size_t* codes_bytes, size_t* scales_bytes);

/* w: bf16 or fp32 [K,N] row-major (w_is_f32 selects).  If `interleave2` != 0 the N columns
 * are the concatenation [gate | up] of two N/2-wide matrices and are stored interleaved in
 * blocks of 16 (gate block, up block, ...) so that TNX_EPI_*_MUL sees matching columns in
 * adjacent tiles.  int4_bound: the integer the group's absmax maps to, scale = bf16(absmax /
 * int4_bound) (ignored for NF4); 7 is this format's definition above, and the parameter is there
 * so that a quantiser with another symmetric bound (7.5, 8: codes still clamp to [-8, 7]) can be
 * mirrored without an ABI change; <= 0 selects 7.  Replaces qwix's quantizer reached from
 * tunix/cli/utils/model.py:51-68. */
int tnx_quantize_pack(void* stream, const void* w, int w_is_f32, int64_t K, int64_t N,
                      int group, int qtype, int interleave2, float int4_bound, uint32_t* codes,
                      uint16_t* scales);

/* Inverse of the packing for tests and export: w_out fp32 [K,N] = w^ (bf16 values). */
int tnx_qw_dequant(void* stream, const uint32_t* codes, const uint16_t* scales, int64_t K,
                   int64_t N, int group, int qtype, int interleave2, float* w_out);

/* Optional second copy of a frozen weight for calls with many rows (512 and more: prefill,
 * compute_per_token_logps): the same values w^ = bf16(bf16(level) * scale), 2 bytes per weight,
 * laid out as the matrix-instruction fragments of the many-row kernel, which then loads them as
 * they are instead of converting codes in its loop (results are bit-identical; the kernel is
 * bound by its instruction mix there, not by the 4x larger weight stream).  288 GB of HBM hold
 * it beside the packed weights: 14 GB for the 7 G linear weights of Llama-3.1-8B.  Pass the copy
 * as tnx_qlinear_desc.w_expanded / tnx_lmhead_desc.w_expanded; calls with few rows ignore it.
 * No counterpart in the reference (XLA materialises a dequantised bf16 W on every call). */
size_t tnx_qw_expanded_bytes(int64_t K, int64_t N);
int tnx_qw_expand(void* stream, const uint32_t* codes, const uint16_t* scales, int64_t K, int64_t N,
                  int group, int qtype, uint16_t* w_expanded /* 16-byte aligned */);
/* The same layout from a dense bf16 matrix w[N][K] (an unquantised or tied lm_head, [V][D]): a
 * log-probability pass over 512 rows or more then runs the head on the many-row kernel
 * (tnx_lmhead_desc.w_expanded next to w_bf16) instead of the 128 x 128 one. */
int tnx_dense_expand(void* stream, const uint16_t* w_bf16, int64_t K, int64_t N, uint16_t* w_expanded);

/* ---------------------------------------------------------------------------------------
 * Quantized linear fused with the LoRA delta:  y = epi( x . dequant(W) + lora_scale * t . B )
 * replaces Einsum.__call__ / nnx.Linear as rewritten by qwix (llama3/model.py:216-218,
 * :461-496; qwen3/model.py:361-365; gemma3/model.py:398-399) and the merge formula
 * W + (A @ B) * alpha / rank pinned at tunix/models/safetensors_saver.py:107.
 * ------------------------------------------------------------------------------------- */
typedef struct tnx_qlinear_desc {
  int64_t M, K, N;          /* N counts packed columns (after interleave2 it is 2*F)        */
  int group, qtype;
  const uint16_t* x;        /* bf16 [M,K]                                                   */
  const uint32_t* codes;    /* QW codes                                                     */
  const uint16_t* scales;   /* QW scales                                                    */
  /* LoRA (optional: lora_rank == 0 disables). t = bf16(x . A) comes from tnx_lora_down.    */
  int lora_rank;            /* r, multiple of 32                                            */
  int lora_nseg;            /* 1..4 column segments, each with its own t columns; -1: the
                               columns are an interleaved gate/up pair (even tiles use t
                               columns [0,r), odd tiles [r,2r))                             */
  int64_t lora_seg_end[4];  /* exclusive end column (packed order) of each segment, %16==0  */
  int lora_seg_toff[4];     /* first t column of each segment                               */
  int64_t t_ld;             /* row stride of t in elements                                  */
  const uint16_t* t;        /* bf16 [M, t_ld]                                               */
  const uint16_t* lora_b;   /* bf16 [N, r] (B transposed: r contiguous)                     */
  float lora_scale;         /* alpha / rank                                                 */
  int epilogue;             /* TNX_EPI_*                                                    */
  const uint16_t* residual; /* bf16 [M, N] for TNX_EPI_RESIDUAL                             */
  void* y;                  /* bf16 [M,N]; *_MUL: bf16 [M,N/2]; TNX_EPI_F32: fp32 [M,N]     */
  int split_k;              /* >1: the K range is split over work-groups, each writing its
                               partial tile into `ws`                                       */
  float* ws;                /* fp32 [split_k, M, N] workspace (need not be initialised);
                               required when split_k > 1; tnx_splitk_finish adds the
                               partial tiles in split order and applies the epilogue        */
  /* Optional (next_tpart != NULL), *_MUL epilogues with split_k == 1 only: the LoRA
   * down-projection of the NEXT linear -- the one that consumes y, e.g. down_proj after
   * gate|up -- fused into this epilogue.  Each (up to) 128-row x 128-column work-group tile leaves
   * its share of y . A_next as one fp32 fragment plane; tnx_lora_reduce adds the planes in a fixed
   * order and writes t_next = bf16(y . A_next), which tnx_lora_down would have produced.    */
  const uint16_t* next_a_t; /* bf16 [next_rank, N/2]: A_next transposed                     */
  int next_rank;            /* multiple of 16, <= 64                                        */
  float* next_tpart;        /* fp32 [ceil(M/128) * ceil(N/128)][8192]                       */
  const uint16_t* w_expanded; /* optional: tnx_qw_expand of (codes, scales); NULL: none       */
} tnx_qlinear_desc;

int tnx_qlinear_lora(void* stream, const tnx_qlinear_desc* h_desc);
/* Epilogue for split_k > 1 (same desc): y = epi(sum_z ws[z]). */
int tnx_splitk_finish(void* stream, const tnx_qlinear_desc* h_desc);

/* t[M, :R] = bf16(sum over the n_col_blocks fragment planes that tnx_qlinear_lora left in
 * tpart through next_tpart), planes added in column-block order. */
int tnx_lora_reduce(void* stream, const float* tpart, int64_t M, int64_t n_col_blocks, int R,
                    uint16_t* t, int64_t t_ld);

/* t[M, R] = bf16( x[M,K] . A ), a_t = A transposed: bf16 [R, K].  R multiple of 16.
 * The LoRA "down" half of qwix's x @ lora_a @ lora_b (shapes at
 * tunix/models/llama3/mapping_sglang_jax.py:64-145). */
int tnx_lora_down(void* stream, const uint16_t* x, int64_t M, int64_t K, const uint16_t* a_t,
                  int R, uint16_t* t, int64_t t_ld);

/* ---------------------------------------------------------------------------------------
 * Embedding gather: out[m,:] = table[ids[m],:] * scale_bf16  (scale 1.0 = plain copy).
 * Embedder.encode llama3/model.py:238-242, qwen3/model.py:390-395, gemma3/model.py:353-358
 * (gemma3 multiplies by bf16(sqrt(D))).  ids are read as ids[row_stride*b + col(+t)].
 * ------------------------------------------------------------------------------------- */
int tnx_embed(void* stream, const uint16_t* table, int64_t V, int64_t D, const int32_t* ids,
              int64_t ids_ld, const int32_t* col_ptr, int64_t B, int64_t T, float scale,
              uint16_t* out);

/* RMSNorm over the last axis, three dtype flows.
 *   h = (res_pre ? bf16(x + res_pre) : x);  if (h_out) h_out = h;
 *   y = norm(h) ;  if (res_post) y = bf16(y + res_post)
 * llama3/model.py:290-297, qwen3/model.py:450-456, gemma3/model.py:940-950; residual adds
 * llama3/model.py:560-563, gemma3/model.py:875-898. */
int tnx_rmsnorm(void* stream, const uint16_t* x, const uint16_t* res_pre, uint16_t* h_out,
                const uint16_t* w, const uint16_t* res_post, uint16_t* y, int64_t M, int64_t D,
                float eps, int flavor);
/* The same, with the input row taken from the fp32 partial planes ws[split_k][M][D] that
 * tnx_qlinear_lora leaves when split_k > 1 (N == D): x = bf16(sum_z ws[z]) in split order.  It
 * replaces tnx_splitk_finish + tnx_rmsnorm for a linear whose output feeds a residual add and a
 * norm (o_proj / down_proj: llama3/model.py:560-563).  D % 8 == 0. */
int tnx_rmsnorm_splitk(void* stream, const float* ws, int split_k, const uint16_t* res_pre,
                       uint16_t* h_out, const uint16_t* w, const uint16_t* res_post, uint16_t* y,
                       int64_t M, int64_t D, float eps, int flavor);
/* The same, with the input row taken from the k routed rows of a token: x = bf16(sum_j topk_w[m,j]
 * * y_route[m*k + j]), j ascending (tnx_moe_combine's arithmetic).  It replaces tnx_moe_combine +
 * tnx_rmsnorm where an MoE layer's output feeds the residual add and the next norm
 * (qwen3/model.py:826-832 into :450-456).  D % 8 == 0. */
int tnx_rmsnorm_moe_combine(void* stream, const uint16_t* y_route, const uint16_t* topk_w, int k,
                            const uint16_t* res_pre, uint16_t* h_out, const uint16_t* w,
                            const uint16_t* res_post, uint16_t* y, int64_t M, int64_t D, float eps,
                            int flavor);
/* Two norms in a row in one launch: y as above (input x, or the partial planes ws of a split-k
 * linear when x is NULL), then y2 = norm(y) with weight w2.  Gemma-3's block applies
 * post_attention_norm, adds the residual and applies pre_ffw_norm to the sum, and likewise
 * post_ffw_norm + residual followed by the next block's pre_attention_norm
 * (gemma3/model.py:882-898): y = h + norm(x) . w is the new residual stream, y2 the next
 * linear's input.  Results equal those of two tnx_rmsnorm launches bit for bit.  D % 8 == 0. */
int tnx_rmsnorm_pair(void* stream, const uint16_t* x, const float* ws, int split_k,
                     const uint16_t* res_pre, uint16_t* h_out, const uint16_t* w,
                     const uint16_t* res_post, uint16_t* y, const uint16_t* w2, uint16_t* y2,
                     int64_t M, int64_t D, float eps, int flavor);

/* ---------------------------------------------------------------------------------------
 * Per-head q/k RMSNorm (optional) + RoPE + KV-cache write for T tokens per row.
 *   qkv: bf16 [B*T, (Hq+2*Hkv)*dh] (q heads, then k heads, then v heads)
 *   positions[b*pos_ld + col + t], col = *col_ptr (device) : RoPE position of token t of row b
 *   cache slot of token t = (*col_ptr + t) % S
 *   q_out: bf16 [B*T, Hq*dh];  kcache/vcache: bf16 [B, Hkv, S, dh]
 * apply_rope llama3/model.py:249-270 (call sites :356-365 never pass rope_theta, so theta is
 * 1e6), qwen3/model.py:404-425 (+ q_norm/k_norm :531-532), gemma3/model.py:402-430 (+ q/k
 * norm :586-587, query pre-scale :596); cache write llama3/model.py:367-377.
 * ------------------------------------------------------------------------------------- */
typedef struct tnx_rope_desc {
  int64_t B, T, S;
  int Hq, Hkv, dh;
  int rope_flavor;           /* TNX_ROPE_*                                                  */
  float rope_scale;          /* gemma3: angles are divided by this scale factor (>= 1)      */
  const float* timescale;    /* fp32 [dh/2] device: theta^(2i/dh), computed once by the host */
  int qk_norm;               /* -1 none, else TNX_NORM_* flavour applied per head to q and k */
  float norm_eps;
  const uint16_t* q_norm_w;  /* bf16 [dh] or NULL                                           */
  const uint16_t* k_norm_w;
  float q_prescale;          /* 0 = none; gemma3 multiplies q by bf16(this) after RoPE      */
  const uint16_t* qkv;
  const int32_t* positions;
  int64_t pos_ld;
  const int32_t* col_ptr;    /* device int32: first token-buffer column of this call        */
  uint16_t* q_out;
  uint16_t* kcache;
  uint16_t* vcache;
  const float* qkv_ws;       /* optional: split_k fp32 partial planes [split_k][B*T][(Hq+2Hkv)*dh]
                                of the qkv linear (tnx_qlinear_lora with finish skipped); the
                                input is then bf16(sum of the planes, in split order) and qkv
                                may be NULL                                                   */
  int split_k;
} tnx_rope_desc;
int tnx_qknorm_rope_kvwrite(void* stream, const tnx_rope_desc* h_desc);
/* sin / cos of positions[b, *col_ptr] / timescale[i], fp32 [B, dh/2] each: the angles of the
 * Llama rotation above for one decode step, shared by all layers (input of the fused mode of
 * tnx_gqa_attn). */
int tnx_rope_table(void* stream, const int32_t* positions, int64_t pos_ld, const int32_t* col_ptr,
                   int64_t B, const float* timescale, int dh, float* sin_out, float* cos_out);

/* ---------------------------------------------------------------------------------------
 * GQA attention over the KV cache for T query tokens per row (T = 1: decode).
 * Query token t of row b sits in cache slot c = *col_ptr + t (the caller keeps *col_ptr + T <=
 * tok_ld, the ids one row of `tokens` holds) and attends slot j iff
 *   j <= c  and  tokens[b*tok_ld + j] != pad_id  and (window == 0 or j > c - window),
 * i.e. the mask of compute_attention_masks (tunix/generate/utils.py:34-58) /
 * make_causal_attn_mask (:61-83) and create_sliding_window_mask (gemma3/model.py:477-496),
 * evaluated from the token buffer instead of a dense [B,T,S] mask.
 * scores: s = bf16(q.k) ; s = bf16(s * bf16(scale)) (scale 0: skip, gemma3 pre-scales q);
 * softmax in fp32, probabilities rounded to bf16 before the PV product, fp32 accumulation,
 * output rounded to bf16 (llama3/model.py:379-396, qwen3/model.py:674-686,
 * gemma3/model.py:618-660).
 *   q: bf16 [B*T, Hq*dh]; out: bf16 [B*T, Hq*dh]; caches bf16 [B,Hkv,S,dh]
 *   Every slot of both caches must hold finite values, also the slots no token was written to
 *   yet (allocate the caches zero-filled): a masked key gets probability exactly 0, but its value
 *   row still enters the P.V product, and 0 * NaN or 0 * Inf would poison the output.
 *   ws: fp32 workspace of tnx_attn_ws_bytes() bytes (only touched when the key range is split)
 * ------------------------------------------------------------------------------------- */
typedef struct tnx_attn_desc {
  int64_t B, T, S;
  int Hq, Hkv, dh;
  float scale;
  int window;
  int32_t pad_id;
  const uint16_t* q;
  const uint16_t* kcache;
  const uint16_t* vcache;
  const int32_t* tokens;
  int64_t tok_ld;
  const int32_t* col_ptr;
  int kv_chunk;              /* keys per work-group when splitting (multiple of 32); 0: no split */
  float* ws;
  uint16_t* out;
  /* Optional fused RoPE + cache write for decode (rope_sin != NULL; needs T == 1,
   * dh == 128, a model without q/k norm and the Llama rotation): the kernel takes the step's
   * q, k and v from the qkv linear's output (finished bf16 `qkv` [B, (Hq+2Hkv)*dh], or its
   * `qkv_split` fp32 partial planes `qkv_ws`), rotates q and k exactly as
   * tnx_qknorm_rope_kvwrite does (with the step's sines / cosines from tnx_rope_table), writes k
   * and v into cache slot *col_ptr and attends them from registers; `q` is not read and that
   * separate launch is not needed. */
  const float* qkv_ws;
  const uint16_t* qkv;
  int qkv_split;
  const float* rope_sin;     /* fp32 [B, dh/2] from tnx_rope_table                           */
  const float* rope_cos;
  /* Optional, packed batches (several sequences per row, compute_per_token_logps with
   * segment_ids, tunix/rl/common.py:260-271, :408-418; qwen3/model.py:622-655): int32
   * [B, tok_ld] segment id of every slot.  When given, slot j is attended iff j <= c (and the
   * window test) and segment_ids[b, j] == segment_ids[b, c]; `tokens` and pad_id are not read
   * (padding is its own segment, as the reference's packed callers arrange it). */
  const int32_t* segment_ids;
} tnx_attn_desc;
size_t tnx_attn_ws_bytes(int64_t B, int64_t T, int64_t S, int Hq, int dh, int kv_chunk);
int tnx_gqa_attn(void* stream, const tnx_attn_desc* h_desc);

/* ---------------------------------------------------------------------------------------
 * Fused lm_head -> fp32 log-softmax statistics, never writing [M,V] logits:
 *   logit[m,v] = f32(bf16( x[m,:] . W[v,:] (+ lora) )) / temperature
 * per row m: best id (first maximal index), best logit, logsumexp, and optionally the logit
 * of a given target id.  compute_final_logits llama3/model.py:688-697; sample_best
 * tunix/generate/sampler.py:151-161; selective_log_softmax tunix/rl/common.py:187-203;
 * compute_chunked_logps :485-571.
 *   head weights: dense bf16 [V,D] (w_bf16 != NULL; also the tied embedding table), or QW
 *   part: fp32 workspace [M, n_vblocks, 4]; n_vblocks from tnx_lmhead_nblocks(V)
 *   logits_out (optional) receives the raw logits f32(bf16(x . W)): neither the temperature nor
 *   the forbidden mask is applied to it (the sampler's logits buffer, sampler.py:724-728)
 * ------------------------------------------------------------------------------------- */
typedef struct tnx_lmhead_desc {
  int64_t M, D, V;
  const uint16_t* x;          /* bf16 [M,D]                                                  */
  const uint16_t* w_bf16;     /* bf16 [V,D] or NULL                                          */
  const uint32_t* codes;      /* QW (K = D, N = V) when w_bf16 == NULL                       */
  const uint16_t* scales;
  int group, qtype;
  int lora_rank;
  const uint16_t* t;          /* bf16 [M, t_ld]                                              */
  int64_t t_ld;
  const uint16_t* lora_b;     /* bf16 [V, r]                                                 */
  float lora_scale;
  float temperature;          /* fp32 logits are divided by this (0 or 1.0 = no scaling)     */
  const int32_t* forbidden;   /* device list of ids forced to -inf, or NULL                  */
  int n_forbidden;
  const int32_t* targets;     /* int32 [M] or NULL                                           */
  float* part;
  int32_t* best_id;           /* int32 [M] or NULL                                           */
  float* best_logp;           /* fp32 [M]: log-softmax at best_id, or NULL                   */
  float* target_logp;         /* fp32 [M]: log-softmax at targets[m], or NULL                */
  float* lse;                 /* fp32 [M] or NULL                                            */
  float* logits_out;          /* fp32 [M,V] or NULL: materialise logits (return_logits /
                                 top-k sampling path)                                       */
  float* part_entropy;        /* fp32 workspace [M, n_vblocks], needed when entropy != NULL  */
  float* entropy;             /* fp32 [M] or NULL: -sum_v p_v log p_v of the (temperature-
                                 scaled) distribution, compute_entropy_from_logits
                                 tunix/rl/common.py:1136-1148                                */
  /* Optional whole-vocabulary categorical draw inside the head (draw_id != NULL): what
   * tnx_sample_topk does for top_p >= 1 without top_k (sample_top_p, sampler.py:119-121),
   * jax.random.categorical over logits / temperature with the noise of fold_in(key, *step),
   * without materialising the logits. */
  float* part_draw;           /* fp32 workspace [M, n_vblocks, 3]                            */
  uint32_t draw_key0, draw_key1;
  int draw_rng_variant;       /* as rng_variant of tnx_sample_topk                           */
  const int32_t* draw_step_ptr;
  int32_t* draw_id;           /* int32 [M]                                                   */
  float* draw_logp;           /* fp32 [M]: log-softmax at the drawn id, or NULL              */
  /* fp32-accumulate reference mode: != 0 keeps the fp32 accumulator as the logit instead of
   * rounding it to bf16 first (the reference's head is a bf16 einsum cast to fp32,
   * llama3/model.py:688-697; this mode is what that einsum would give with an fp32 result).
   * Inputs are what they are in the normal mode (bf16 x, weights dequantised to bf16, bf16 t);
   * every sum and the log-softmax run in fp32.  Log-probabilities then agree with an fp64
   * evaluation of the same bf16 operands to 1e-4 instead of to bf16 resolution. */
  int logits_fp32;
  const uint16_t* w_expanded; /* optional: tnx_qw_expand of (codes, scales), or
                                 tnx_dense_expand of w_bf16                                   */
  /* > 0: a logit is softcap * tanh(w . x / softcap), formed in fp32 before it is rounded */
  float softcap;
} tnx_lmhead_desc;
int64_t tnx_lmhead_nblocks(int64_t V);
int tnx_lmhead_logp(void* stream, const tnx_lmhead_desc* h_desc);

/* Top-k / top-p sampling from materialised raw fp32 logits, which are divided by `temperature`
 * on the fly: sample_top_p tunix/generate/sampler.py:105-148.  `forbidden` ids (may be NULL) are
 * treated as -inf (:490-491).  The k largest logits per row (descending,
 * lower index first among equals) are softmaxed, entries whose exclusive cumulative
 * probability exceeds top_p are dropped, and one is drawn by Gumbel-max (jax.random.categorical)
 * with noise from threefry2x32 keyed by fold_in((key0,key1), *step_ptr) (sampler.py:516).
 * rng_variant selects jax's random_bits layout: 1 = partitionable (counter (0,n), x0^x1),
 * 0 = original (counter array split in halves).  k <= 0 (no top-k) with top_p >= 1 draws from
 * the whole vocabulary, noise indexed by vocabulary id (:118-121).  logp_out = full-vocabulary
 * log-softmax at the drawn id (:141-144).
 * 0 < k < V: k <= 1024.  With a workspace `ws` of tnx_sample_topk_ws_bytes(M, V, k) bytes (and
 * ceil(V / 8192) * k <= 4096, k <= 512) the row is processed in segments by many work-groups and a merging
 * launch; with ws = NULL one work-group per row does everything.  Both give the same result.
 * k <= 0 with top_p < 1, and k == V with any top_p, sort every row completely, as the reference
 * does with jax.lax.top_k(k = V) (:126-127), draw over SORTED positions, and need ws of
 * tnx_sample_fullsort_ws_bytes(M, V) bytes (two pairs of [M, V] key / id arrays for the library's
 * own stable radix sort; M * V < 2^31).  k > V returns TNX_EINVAL
 * (jax.lax.top_k raises). */
size_t tnx_sample_topk_ws_bytes(int64_t M, int64_t V, int k);
size_t tnx_sample_fullsort_ws_bytes(int64_t M, int64_t V);
int tnx_sample_topk(void* stream, const float* logits, int64_t M, int64_t V, int k, float top_p,
                    float temperature, uint32_t key0, uint32_t key1, int rng_variant,
                    const int32_t* forbidden, int n_forbidden, const int32_t* step_ptr, float* ws,
                    int32_t* ids_out, float* logp_out);

/* The same draw for 0 < k < V straight after a tnx_lmhead_logp call over the same rows, in one
 * launch that reads k x 128 logits per row instead of the row: the k best logits of a row lie in
 * the k blocks of 128 columns with the largest block maxima, which the head has left in its
 * workspace.  `logits` is that call's logits_out, `part` its workspace, `lse` its lse output
 * (needed when logp_out is given); the call must have used the same `temperature` and the same
 * `forbidden` list.  Ids are those of tnx_sample_topk on the same logits; logp_out is taken
 * against the head's log-sum-exp (the two sum the row's exponentials in different orders).
 * Shapes: tnx_sample_topk_head_ok(V, k) != 0, i.e. k <= 64 and V <= 524288; otherwise TNX_EINVAL
 * and the caller uses tnx_sample_topk.  No workspace. */
int tnx_sample_topk_head_ok(int64_t V, int k);
int tnx_sample_topk_head(void* stream, const float* logits, const float* part, const float* lse,
                         int64_t M, int64_t V, int k, float top_p, float temperature, uint32_t key0,
                         uint32_t key1, int rng_variant, const int32_t* forbidden, int n_forbidden,
                         const int32_t* step_ptr, int32_t* ids_out, float* logp_out);

/* Sampler bookkeeping of one step (tunix/generate/sampler.py:529-535, :692-703):
 *   col = *step_ptr; tokens[b, col+1] = ids[b]; logprobs[b, col+1] = logp[b] (if given);
 *   done[b] |= ids[b] in eos[];  then *step_ptr = col + 1 (by the last thread). */
int tnx_sample_commit(void* stream, const int32_t* ids, const float* logp, int64_t B,
                      int32_t* tokens, int64_t tok_ld, float* logprobs, int32_t* done,
                      const int32_t* eos, int n_eos, int32_t* step_ptr);

/* ---------------------------------------------------------------------------------------
 * MoE (qwen3/model.py:787-832): router softmax -> top-k -> renormalise (weights bf16), and an
 * int4/NF4 grouped GEMM over routed tokens (operator shape of megablox.gmm, :975-995).
 * ------------------------------------------------------------------------------------- */
/* scores: bf16 [M,E] router outputs.  topk_w: bf16 [M,k]; topk_id: int32 [M,k] (descending
 * probability, lower expert id first among equals).  A row with a NaN score still gets k distinct
 * ids inside [0,E) (so that the sort and the grouped GEMM stay in bounds) and NaN weights. */
int tnx_moe_route_topk(void* stream, const uint16_t* scores, int64_t M, int E, int k,
                       uint16_t* topk_w, int32_t* topk_id);
/* Builds the expert-sorted route list: counts[E], offsets[E+1], sorted_route[M*k] (route =
 * m*k + j), stable in route order.  M*k <= 1<<20. */
int tnx_moe_sort_routes(void* stream, const int32_t* topk_id, int64_t M, int k, int E,
                        int32_t* counts, int32_t* offsets, int32_t* sorted_route);
typedef struct tnx_moe_gmm_desc {
  int64_t n_routes;          /* M*k                                                          */
  int E, k;
  int64_t K, N;              /* per-expert linear: x[.,K] . W_e[K,N]                          */
  int group, qtype;
  const uint16_t* x;         /* bf16 rows; row of route r is r / x_div (x_div = k for the
                                token activations, 1 for per-route activations)             */
  int x_div;
  const uint32_t* codes;     /* QW per expert, expert stride = tnx_qw_sizes().codes_bytes    */
  const uint16_t* scales;
  const int32_t* offsets;    /* int32 [E+1]                                                  */
  const int32_t* sorted_route;
  int epilogue;              /* TNX_EPI_STORE or TNX_EPI_SILU_MUL (interleave2 packing)      */
  uint16_t* y;               /* bf16 [n_routes, N or N/2], indexed by route                  */
} tnx_moe_gmm_desc;
int tnx_moe_int4_gmm(void* stream, const tnx_moe_gmm_desc* h_desc);
/* out[m,:] = bf16( sum_j f32(topk_w[m,j]) * f32(y[m*k+j,:]) )  (qwen3/model.py:827-832). */
int tnx_moe_combine(void* stream, const uint16_t* y, const uint16_t* topk_w, int64_t M, int k,
                    int64_t D, const uint16_t* residual, uint16_t* out);

/* GRPO clipped ratio (tunix/rl/algo_core.py:440-489): lr = clip(logp - old, -20, 20);
 * ratio = exp(lr); loss = max(-A*ratio, -A*clip(ratio, 1-eps_lo, 1+eps_hi)).
 * adv has one value per sequence: adv[n / tokens_per_seq].  Outputs may be NULL. */
int tnx_grpo_ratio(void* stream, const float* logp, const float* old_logp, const float* adv,
                   int64_t N, int64_t tokens_per_seq, float eps_lo, float eps_hi, float* ratio,
                   float* loss, int32_t* clipped);

/* Per-token KL estimators between the trained and the reference policy
 * (tunix/rl/common.py:135-184): TNX_KL_KL logp - ref; TNX_KL_MSE 0.5 * (logp - ref)^2;
 * TNX_KL_LOW_VAR exp(d) - d - 1 with d = ref - logp.  clamp >= 0 clips the result to
 * [-clamp, clamp]; a negative clamp means none (the reference's clamp_value=None). */
enum { TNX_KL_KL = 0, TNX_KL_MSE = 1, TNX_KL_LOW_VAR = 2 };
int tnx_kl_divergence(void* stream, const float* logp, const float* ref_logp, int64_t N, int method,
                      float clamp, float* kl);

/* Loss aggregation without packing segments (tunix/rl/common.py:763-854, the per-row branch): out[0] = unreduced sum,
 * out[1] = denominator of the mode; the caller divides as WeightedMetric.compute does
 * (tunix/sft/utils.py:201-219).  per_token_loss, mask: fp32 [B, T]; row_ws: [B, 2] fp32 workspace
 * (per-row sum of loss * mask, per-row sum of mask).  norm: the `norm` keyword of the two modes
 * that take one (the caller passes the reference's default, T or B, when the keyword is absent).
 * Sums run in a fixed order: the result is the same on every launch. */
enum {
  TNX_AGG_TOKEN_MEAN = 0,              /* "token-mean" */
  TNX_AGG_SEQ_MEAN_TOKEN_MEAN = 1,     /* "sequence-mean-token-mean" */
  TNX_AGG_SEQ_MEAN_TOKEN_SCALE = 2,    /* "sequence-mean-token-scale" */
  TNX_AGG_SEQ_MEAN_TOKEN_SUM = 3,      /* "seq-mean-token-sum" */
  TNX_AGG_SEQ_MEAN_TOKEN_SUM_NORM = 4  /* "sequence-mean-token-sum-norm" */
};
int tnx_aggregate_loss(void* stream, const float* per_token_loss, const float* mask, int64_t B, int64_t T,
                       int mode, float norm, float* row_ws, float* out);

/* The same over packed batches (the segment branch, tunix/rl/common.py:857-940 with the segment
 * sums of :704-760): a row holds several sequences, segment_ids int32 [B, T] tells them apart
 * (0 = padding, ids outside [0, num_segments) belong to no segment), and the per-sequence modes
 * reduce per segment: a segment counts when it has at least one token with mask != 0, segment 0
 * never counts, the denominator is the number of counted segments.  "token-mean" and
 * "sequence-mean-token-sum-norm" sum over all tokens as without packing; norm <= 0 in the latter
 * selects the reference's default there, the number of counted segments.
 * "sequence-mean-token-scale" needs an explicit norm > 0.  ws: tnx_aggregate_loss_segmented_ws_bytes
 * bytes.  Every sum runs in a fixed order. */
size_t tnx_aggregate_loss_segmented_ws_bytes(int64_t B, int num_segments);
int tnx_aggregate_loss_segmented(void* stream, const float* per_token_loss, const float* mask,
                                 const int32_t* segment_ids, int64_t B, int64_t T, int num_segments,
                                 int mode, float norm, float* ws, float* out);

/* Agreement between the log-probabilities the rollout recorded and the ones the trainer
 * recomputes for the same tokens (tunix/rl/grpo/grpo_learner.py:405-440), over the positions
 * where mask != 0.  rollout_logp, trainer_logp, mask: fp32 [B, T].  out5 = { mean |dlogp|,
 * max |dlogp|, mean |dp|, max |dp|, Pearson correlation of the probabilities } with
 * p = exp(logp), means over max(mask count, 1), correlation = cov / sqrt(max(var_r * var_t, 1e-12)).
 * ws: tnx_logp_drift_ws_bytes(B) bytes, 8-byte aligned.  The moments are accumulated in double. */
size_t tnx_logp_drift_ws_bytes(int64_t B);
int tnx_logp_drift(void* stream, const float* rollout_logp, const float* trainer_logp, const float* mask,
                   int64_t B, int64_t T, void* ws, float* out5);

/* tnx_logp_drift for callers that cannot allocate device memory (code under HIP-graph capture,
 * tight serving loops, harnesses that forbid hipMalloc): no counterpart in the reference.  Same
 * arguments and results as tnx_logp_drift without the workspace: the per-row moments go to an
 * array built into the library (tnx_logp_drift_static_max_rows() = 4096 rows, 320 KiB, one copy
 * per GPU for the life of the process).  B above that limit returns TNX_EINVAL.  The call
 * allocates and frees nothing; its first call on a device looks the array's address up
 * (hipGetSymbolAddress), so make that call outside a capture.  Every call on one GPU shares
 * that GPU's array: calls that overlap on one GPU (different streams, no ordering) race. */
int64_t tnx_logp_drift_static_max_rows(void);
int tnx_logp_drift_static(void* stream, const float* rollout_logp, const float* trainer_logp,
                          const float* mask, int64_t B, int64_t T, float* out5);

/* Fill n 32-bit words with `value` (graph-capturable replacement for hipMemsetAsync). */
int tnx_fill_u32(void* stream, uint32_t* p, int64_t n, uint32_t value);

/* ---------------------------------------------------------------------------------------
 * Decoders with dense weights and an fp32 residual stream.  They have no counterpart in the
 * reference tree; each entry point is one mechanism with its constants as arguments.
 *
 * dtype: the model's: TNX_BF16 (matrix operands bf16, fp32 accumulation) or TNX_F32 (everything
 * fp32).  The residual, norms, angles, scores, softmax and recurrent states are fp32 in both.
 * A sequence of batch row b occupies the columns starts[b], starts[b] + 1, ... of its row (left
 * padding in front of it); its position counts from 0 at starts[b].  *col_ptr is the column of the
 * call's first token.
 * Fragment order (x_frag / y_frag / out_frag = 1, bf16): activations in blocks of 32 rows x 16
 * columns, inside a block [column / 8][row][column % 8]; what tnx_dense_linear reads fastest at few
 * rows.  Buffers hold whole blocks of 128 rows.
 */
#define TNX_BF16 0
#define TNX_F32 1

/* Rows of a linear's output: y (model dtype), or with split_k > 1 the fp32 partial planes
 * ws[z * plane + row * ld + col] to be summed in z order. */
typedef struct {
  const void* y;
  const float* ws;
  int split_k;
  int64_t plane;
  int64_t ld;
} tnx_rows_src;

/* y[M, N] = x[M, K] . w^T.  bf16: w is the fragment-order copy of tnx_dense_expand, K % 128 == 0
 * (zero-padded), N % 16 == 0 for bf16 outputs.  fp32: w row-major [N, K], K % 16 == 0.
 * epilogue: TNX_EPI_STORE or TNX_EPI_RELU2 (model dtype; the square of the positive part, formed in fp32), TNX_EPI_F32, or (bf16) TNX_EPI_GELU_MUL / TNX_EPI_SILU_MUL: w's
 * rows come in alternating blocks of 16 gate and 16 up rows and y[M, N/2] = act(gate) * up with act =
 * gelu_tanh / silu, formed in fp32 and rounded once.  split_k > 1 (bf16, few rows): fp32 planes to ws
 * [split_k][M][ldy] instead.
 * batch > 1: the same for z = 0 .. batch - 1 with x, w and y moved on by z times their strides.
 * n_experts > 0: M counts routes; route r of expert e (sorted_route[offsets[e] .. offsets[e + 1])) reads row
 * r / x_div of x and weight e (w + e * w_stride) and writes row r of y. */
typedef struct {
  int64_t M, K, N;
  int dtype;
  const void* x;
  int64_t ldx;
  int x_frag;
  const void* w;
  int epilogue;
  void* y;
  int64_t ldy;
  int y_frag;
  int split_k;
  float* ws;
  int64_t batch;
  int64_t x_stride, w_stride, y_stride;   /* elements */
  int n_experts, x_div;
  const int32_t* offsets;                 /* [n_experts + 1] */
  const int32_t* sorted_route;            /* [M] */
} tnx_dense_desc;
int tnx_dense_linear(void* stream, const tnx_dense_desc* d);

/* x[row] (fp32) = scale * table[ids[b, col + t]]; optionally also cat[row, cat_off ..] = the table's row in the
 * model's dtype.  Ids outside [0, V) read row 0.  pos (null: none; [n_pos, D] in the table's dtype): pos[p] is added,
 * unscaled, p = the token's position col + t - starts[b], held inside the table (the caller bounds sequences). */
int tnx_embed_rows(void* stream, int dtype, const void* table, int64_t V, int64_t D, const int32_t* ids,
                   int64_t ids_ld, const int32_t* col_ptr, int64_t B, int64_t T, float scale, float* x, void* cat,
                   int64_t cat_ld, int64_t cat_off, int cat_frag, const void* pos, int64_t n_pos, const int32_t* starts);

/* The residual step between two sublayers, in fp32:
 *   mode 1: x += norm(y) * (w_offset + w_post);  mode 2: x = y;  mode 3: x = norm(x) * (w_offset + w_post);
 *   mode 0: x stays;
 *   out (model dtype) = norm(x) * (w_offset + w_next), or x itself when w_next is null,
 * with norm(v) = v / sqrt(mean(v^2) + eps), over each of `groups` equal parts of the row (0: one part).  y.ws
 * with split_k >= 1: fp32 planes.  x_out (null: x) takes the new x.
 * route_w (null: none): y holds route_k rows per row of x, which are summed with the weights route_w[row, :].
 * shift (null: none; instead of w_next): out = x + (x' - x) * shift with x' the x of the token before: the row in
 * front of it, or `before` [B, D] for the first token of a call (zeros for the first token of a sequence).  The
 * rows are T tokens for each of B sequences.  T == 1: `before` takes the new x; T > 1: x_out is another
 * buffer than x, and the caller keeps the last rows (tnx_ring_write).
 * center: norms are layer norms, (v - mean) / sqrt(mean((v - mean)^2) + eps).  mult (0: 1): mode 1 adds mult * norm(y).
 * extra (extra.ld 0: none): rows that join y before its norm, times extra_w[row] (null: 1).
 * hist (null: none): the results of earlier layers, X_j at hist + j * hist_plane, j < hist_n.  The new x is X_n
 * (n = hist_n): it is stored there when hist_store is set, and x becomes sum_{j <= n} hist_w[j] X_j.  These four go with
 * modes 0 and 1, one part and no shift. */
typedef struct {
  int64_t M, D;
  int dtype;
  float eps, w_offset;
  int mode;
  tnx_rows_src y;
  const float* w_post;
  float* x;
  const float* w_next;
  void* out;
  int64_t out_ld;
  int out_frag;
  int groups;
  float* x_out;
  const float* route_w;
  int route_k;
  const float* shift;
  float* before;
  const int32_t* starts;
  const int32_t* col_ptr;
  int64_t B, T;
  int center;
  float mult;
  tnx_rows_src extra;
  const float* extra_w;
  float* hist;
  int64_t hist_plane;
  int hist_n, hist_store;
  const float* hist_w;   /* [hist_n + 1] */
} tnx_residual_norm_desc;
int tnx_residual_norm(void* stream, const tnx_residual_norm_desc* d);

/* Rotation of the first rot_dims dimensions of every query and key head (pairs (i, i + rot_dims/2),
 * angle position * inv_freq[i] in fp32) and the cache write.  y: q heads from column 0, k from k_off,
 * v from v_off.  q_out [B*T, H, dkp]; kcache [B, G, S, dkp], vcache [B, G, S, dvp] at slot col + t;
 * dimensions past dk / dv are written as zeros. */
typedef struct {
  int64_t B, T, S;
  int H, G, dk, dv, dkp, dvp, rot_dims;
  int dtype;
  const float* inv_freq;
  tnx_rows_src y;
  int64_t k_off, v_off;
  const int32_t* starts;
  const int32_t* col_ptr;
  void* q_out;
  void* kcache;
  void* vcache;
} tnx_part_rope_desc;
int tnx_part_rope_kvwrite(void* stream, const tnx_part_rope_desc* d);

/* Query and key norms over a whole projection and the cache write: q and k are divided by the root mean square of all
 * their heads together (eps inside the root) times w_q [H * dk] and w_k [G * dk]; the rest as tnx_part_rope_kvwrite.
 * kcache null: q alone (keys and values are another layer's). */
typedef struct {
  int64_t B, T, S;
  int H, G, dk, dv, dkp, dvp;
  int dtype;
  float eps;
  const float* w_q;
  const float* w_k;
  tnx_rows_src y;
  int64_t k_off, v_off;
  const int32_t* col_ptr;
  void* q_out;
  void* kcache;
  void* vcache;
} tnx_rownorm_kvwrite_desc;
int tnx_rownorm_kvwrite(void* stream, const tnx_rownorm_kvwrite_desc* d);

/* Causal attention over keys starts[b] .. col + t with softmax(scale * q.k) whose denominator also
 * holds exp(sinks[head]) (sinks null: none).  out[row, head * out_head ..] (out_head 0: dv).  kv_chunk > 0 splits the key range (few
 * query rows, workspace of tnx_sink_attn_ws_bytes).  slopes (null: none; [H]): slopes[head] times the distance of the
 * two positions is taken off a score.  chunk > 0: a position sees the keys of its own chunk alone, chunks of that many
 * positions counted from starts[b].  tnx_sink_attn_pad: the padded head size the
 * MFMA kernels take (other sizes, and fp32, run a plain kernel). */
typedef struct {
  int64_t B, T, S;
  int H, G, dk, dv, dkp, dvp;
  float scale;
  int dtype;
  const void* q;
  const void* kcache;
  const void* vcache;
  const float* sinks;
  const int32_t* starts;
  const int32_t* col_ptr;
  int kv_chunk;
  float* ws;
  void* out;
  int64_t out_ld;
  int out_frag;
  int64_t out_head;
  const float* slopes;
  int chunk;
} tnx_sink_attn_desc;
int tnx_sink_attn_pad(int dim, int is_value);
size_t tnx_sink_attn_ws_bytes(int64_t B, int64_t T, int64_t S, int H, int dvp, int kv_chunk);
int tnx_sink_attn(void* stream, const tnx_sink_attn_desc* d);

/* Lightning attention: S <- decay[h] S + k v^T, o = S^T q per head, with q, k, v = silu of y's columns
 * (q from 0, k from k_off, v from v_off; head by head).  state fp32 [B, H, dk, dv] is read unless
 * col <= starts[b] and written back; o fp32 [B*T, o_ld]. */
typedef struct {
  int64_t B, T;
  int H, dk, dv;
  int dtype;
  const float* decay;
  tnx_rows_src y;
  int64_t k_off, v_off;
  const int32_t* starts;
  const int32_t* col_ptr;
  float* state;
  float* o;
  int64_t o_ld;
  float* ws;
} tnx_lightning_desc;
size_t tnx_lightning_ws_bytes(int64_t B, int64_t T, int H, int dk, int dv);
int tnx_lightning(void* stream, const tnx_lightning_desc* d);

/* Linear attention with a forget gate per channel, whose complement writes (HGRN2): per head
 *   f = lower + (1 - lower) sigmoid(z + bias),  S <- diag(f) S + (1 - f) v^T,  o = S^T silu(q)
 * with q and v columns of y (from q_off and v_off, head by head) and z of the fp32 rows f (from f_off); bias and lower
 * [H * dk].  y_f32: y's finished rows are fp32, whatever dtype says (planes always are).  state fp32 [B, H, dk, dv] is read
 * unless col <= starts[b] and written back; o fp32 [B*T, o_ld].
 * norm_w (null: none; [dv], T == 1 and tnx_gated_state_step_ok): heads are divided by their root mean square, times norm_w,
 * and leave in out (model dtype) instead. */
typedef struct {
  int64_t B, T;
  int H, dk, dv;
  int dtype, y_f32;
  tnx_rows_src y;
  int64_t q_off, v_off;
  tnx_rows_src f;
  int64_t f_off;
  const float* bias;
  const float* lower;
  const int32_t* starts;
  const int32_t* col_ptr;
  float* state;
  float* o;
  int64_t o_ld;
  float* ws;
  const float* norm_w;
  float eps;
  void* out;
  int64_t out_ld;
  int out_frag;
} tnx_gated_state_desc;
int tnx_gated_state_step_ok(int dk, int dv);
size_t tnx_gated_state_ws_bytes(int64_t B, int64_t T, int H, int dk, int dv);
int tnx_gated_state(void* stream, const tnx_gated_state_desc* d);

/* out = norm(o) * (w_offset + w) * sigmoid(g[:, g_off ..]), gate_first: out = norm(o * silu(g[:, g_off ..])) *
 * (w_offset + w), the norms over each of `groups` equal parts of a row of W values (0: one).  g.ld 0: no gate.
 * shared_w: w holds one part's weights, for every part. */
typedef struct {
  int64_t M, W;
  int dtype;
  float eps, w_offset;
  const float* o;
  int64_t o_ld;
  tnx_rows_src g;
  int64_t g_off;
  const float* w;
  void* out;
  int64_t out_ld;
  int out_frag;
  int gate_first, groups;
  int shared_w;
} tnx_gated_norm_desc;
int tnx_gated_norm(void* stream, const tnx_gated_norm_desc* d);

/* out[M, F] = gelu_tanh(y[:, :F]) * y[:, up_off : up_off + F]. */
int tnx_gelu_mul(void* stream, int dtype, const void* y, int64_t ld, int64_t up_off, int64_t M, int64_t F,
                 void* out, int64_t out_ld);
/* The same with silu. */
int tnx_silu_mul(void* stream, int dtype, const void* y, int64_t ld, int64_t up_off, int64_t M, int64_t F,
                 void* out, int64_t out_ld);

/* Choice of experts from fp32 logits z [M, E] (z.y fp32, or planes): topk_id int32 [M, k], the k largest logits in
 * descending order (lower id first among equals); topk_w fp32 [M, k], the softmax over these k alone. */
int tnx_route_softmax(void* stream, const tnx_rows_src* z, int64_t M, int E, int k, float* topk_w, int32_t* topk_id);
/* The same with scores s = softmax over all E logits: the k experts with the largest s + correction (correction [E], null:
 * none) are chosen; topk_w = s / (sum of the chosen s + 1e-20) * scale.  gate_w (null: none) fp32 [M] = sigmoid of z's column
 * gate_off.  ld: entries of a row of topk_w and topk_id; those from k on are the experts E, E + 1, .. with that sigmoid as
 * their weight (experts that all rows use). */
int tnx_route_scores(void* stream, const tnx_rows_src* z, int64_t M, int E, int k, const float* correction, float scale, int64_t gate_off,
                     int ld, float* topk_w, int32_t* topk_id, float* gate_w);

/* out[M, F] = a norm(y) + b norm(y^2) + c norm(y^3) + e with norm(v) = v / sqrt(mean(v^2) + eps) over the F values of a row,
 * powers element by element; coef [4] = a, b, c, e. */
int tnx_poly_norm(void* stream, int dtype, const tnx_rows_src* y, int64_t M, int64_t F, const float* coef, float eps, void* out,
                  int64_t out_ld, int out_frag);

/* Causal convolution per channel and silu: out[row, c] = silu(bias[c] + sum_j w[taps - 1 - j, c] u(t - j, c)) for
 * the channels off .. off + C - 1 of y.  Tokens before the call's first one come from the ring [B, slots, C] (model
 * dtype, slot = column % slots, slots >= taps - 1); before starts[b] lie zeros.  The ring is not written. */
typedef struct {
  int64_t B, T, C;
  int taps, slots;
  int dtype;
  tnx_rows_src y;
  int64_t off;
  const float* w;
  const float* bias;
  const void* ring;
  const int32_t* starts;
  const int32_t* col_ptr;
  void* out;
  int64_t out_ld;
} tnx_short_conv_desc;
int tnx_short_conv(void* stream, const tnx_short_conv_desc* d);
/* ring[b, (col + t0 + t) % slots, :] = y[b * T + t, off .. off + C) for the last min(T, slots) tokens. */
int tnx_ring_write(void* stream, int dtype, const tnx_rows_src* y, int64_t off, int64_t B, int64_t T, int64_t C, int slots,
                   const int32_t* col_ptr, int64_t t0, void* ring);

/* State-space duality: per head h (group h / (H / G)), dt = softplus(y[:, dt_off + h] + dt_bias[h]),
 *   S <- exp(-exp(A_log[h]) dt) S + dt B x^T,  o[row, h * P ..] = S^T C + D[h] x.
 * u: convolved rows (model dtype): x [H, P] from column 0, B [G, N] behind it, C [G, N] behind that.  u null, T == 1 and
 * tnx_ssd_step_ok: x, B and C are formed from y's channels c_off .. with the convolution of tnx_short_conv
 * (slots >= taps), whose ring takes the current inputs.  state fp32 [B, H, N, P] is read unless col <= starts[b] and
 * written back; o fp32.  ws: tnx_ssd_ws_bytes. */
typedef struct {
  int64_t B, T;
  int H, G, N, P;
  int dtype;
  const float* A_log;
  const float* dt_bias;
  const float* D;
  tnx_rows_src y;
  int64_t dt_off;
  const void* u;
  int64_t u_ld;
  int64_t c_off;
  int taps, slots;
  const float* conv_w;
  const float* conv_b;
  void* ring;
  const int32_t* starts;
  const int32_t* col_ptr;
  float* state;
  float* o;
  int64_t o_ld;
  float* ws;
} tnx_ssd_desc;
int tnx_ssd_step_ok(int N, int P);
size_t tnx_ssd_ws_bytes(int64_t B, int64_t T, int H, int G, int N, int P);
int tnx_ssd(void* stream, const tnx_ssd_desc* d);

/* Attention through a latent.  A position's cache row (model dtype, `row` elements): its latent c [rank], zeros to
 * rank_pad = rank rounded up to 16, the rotated key part [rot] that all heads share, zeros to row.  tnx_latent_row: the row
 * length to use.
 * tnx_latent_prep: q_out = norm(y[:, q_off .. + q_rank]) * w_q, c = norm(y[:, kv_off .. + rank]) * w_kv (also to c_out
 * unless null), the rot columns behind it rotated (pairs (2i, 2i + 1), angle position * inv_freq[i]), cache row at slot
 * col + t. */
typedef struct {
  int64_t B, T, S;
  int q_rank, rank, rot, rank_pad, row;
  int dtype;
  float eps;
  tnx_rows_src y;
  int64_t q_off, kv_off;
  const float* w_q;
  const float* w_kv;
  const float* inv_freq;
  const int32_t* starts;
  const int32_t* col_ptr;
  void* q_out;
  int64_t q_ld;
  int q_frag;
  void* c_out;
  int64_t c_ld;
  int c_frag;
  void* cache;
} tnx_latent_prep_desc;
int tnx_latent_row(int rank, int rot, int dtype);
int tnx_latent_prep(void* stream, const tnx_latent_prep_desc* d);
/* Heads of y ([n unrotated, r rotated] each): un[row, head * un_ld ..] = the first n and zeros to un_pad,
 * rot[row, head * rot_ld ..] = the last r, rotated as above, and zeros to rot_pad. */
typedef struct {
  int64_t B, T;
  int H, n, r;
  int dtype;
  tnx_rows_src y;
  const float* inv_freq;
  const int32_t* starts;
  const int32_t* col_ptr;
  void* un;
  int64_t un_ld;
  int un_pad;
  void* rot;
  int64_t rot_ld;
  int rot_pad;
} tnx_latent_q_desc;
int tnx_latent_q(void* stream, const tnx_latent_q_desc* d);
/* Operands of tnx_sink_attn for the first T columns: k [B, H, T, dkp] = [y's n columns of the head | the cache row's
 * rotated part], v [B, H, T, dvp] = y's vd columns of the head from v_off on; zeros behind. */
typedef struct {
  int64_t B, T, S;
  int H, n, r, vd, dkp, dvp, rank_pad, row;
  int dtype;
  tnx_rows_src y;
  int64_t v_off;
  const void* cache;
  void* k;
  void* v;
} tnx_latent_kv_desc;
int tnx_latent_kv(void* stream, const tnx_latent_kv_desc* d);
/* bf16: q [B * T, H, row] against the cache rows of columns starts[b] .. col + t, softmax(scale * q . row), out[row, head]
 * [out_head] = the weighted sum of the rows' first `rank` elements.  kv_chunk > 0 (a multiple of 64) splits the key
 * range (workspace of tnx_latent_attn_ws_bytes).  Rows of other lengths, and fp32: tnx_sink_attn with one kv head whose
 * keys and values are the cache rows. */
typedef struct {
  int64_t B, T, S;
  int H, rank, row;
  float scale;
  const void* q;
  const void* cache;
  const int32_t* starts;
  const int32_t* col_ptr;
  int kv_chunk;
  float* ws;
  void* out;
  int64_t out_head;
} tnx_latent_attn_desc;
int tnx_latent_attn_ok(int rank, int row, int64_t S);
size_t tnx_latent_attn_ws_bytes(int64_t B, int64_t T, int64_t S, int H, int rank, int kv_chunk);
int tnx_latent_attn(void* stream, const tnx_latent_attn_desc* d);

/* out[row, i] = y[row * y_ld + (i / head) * y_head + i % head] * sigmoid(g[row, g_off + i]), i < W. */
typedef struct {
  int64_t M, W;
  int head;
  int dtype;
  const void* y;
  int64_t y_ld, y_head;
  tnx_rows_src g;
  int64_t g_off;
  void* out;
  int64_t out_ld;
  int out_frag;
} tnx_gate_mul_desc;
int tnx_gate_mul(void* stream, const tnx_gate_mul_desc* d);

/* The step between layers whose sublayers read one norm, in fp32:
 *   x += mult * sum_p y_scale[p] * (w_post[p] ? norm(y[p]) * w_post[p] : y[p]),   then x += add[:] (null: nothing);
 *   h = norm(x) * w_next,   out1 = h + conv1(h),  out2 = h + conv2(h)   (model dtype)
 * over n_in (0 .. 3) incoming rows, norm(v) = v / sqrt(mean(v^2) + eps), conv(h)_t = sum_j w[taps - 1 - j, :] h_(t - j) with
 * zeros before starts[b] (w [taps, D]; conv1 null: out1 = h, taps is then not read; out2 null: not written).  The rows
 * are T tokens for each of B sequences; h of the columns before the call is read from the ring fp32 [B, slots, D]
 * (slot = column % slots, slots >= taps - 1).  x_out takes the new x; null: x stays as it is (n_in == 0, add null).
 * T == 1: the ring takes h, x_out may be x.  T > 1 and taps > 1: x_out is another buffer than x, and `tail` fp32
 * [B, min(T, taps - 1), D] takes h of the last tokens, which the caller moves to the ring (tnx_ring_write). */
typedef struct {
  int64_t M, D;
  int dtype;
  float eps, mult;
  int n_in;
  tnx_rows_src y[3];
  const float* w_post[3];
  float y_scale[3];
  float* x;
  float* x_out;
  const float* add;
  const float* w_next;
  int taps, slots;
  const float* conv1;
  const float* conv2;
  void* out1;
  void* out2;
  int64_t out_ld;
  int out_frag;
  float* ring;
  float* tail;
  const int32_t* starts;
  const int32_t* col_ptr;
  int64_t B, T;
} tnx_parallel_step_desc;
int tnx_parallel_step(void* stream, const tnx_parallel_step_desc* d);

/* Causal convolution per channel of projected q, k and v, then: q times 1 + temp_coef * ln(floor((p + 1) /
 * temp_every) + 1) at position p (temp_coef 0: nothing); each value head divided by sqrt(mean(v^2) + eps) with
 * value_norm; cache write at slot col + t.  y's channels off .. off + C - 1 hold q heads from q_off, k from k_off, v
 * from v_off (offsets from `off`); w [taps, C] fp32, the last row for the current token; ring (model dtype) [B, slots, C],
 * zeros before starts[b].  T == 1: slots >= taps, the ring takes the current channels; T > 1: it is only read.
 * q_out [B*T, H, dkp], kcache [B, G, S, dkp], vcache [B, G, S, dvp]; dimensions past dk / dv are written as zeros. */
typedef struct {
  int64_t B, T, S;
  int H, G, dk, dv, dkp, dvp;
  int taps, slots, dtype;
  float temp_coef, temp_every, eps;
  int value_norm;
  tnx_rows_src y;
  int64_t off, C, q_off, k_off, v_off;
  const float* w;
  void* ring;
  const int32_t* starts;
  const int32_t* col_ptr;
  void* q_out;
  void* kcache;
  void* vcache;
} tnx_conv_kvwrite_desc;
int tnx_conv_kvwrite(void* stream, const tnx_conv_kvwrite_desc* d);

/* Causal attention whose softmax weights are mixed between the heads: with p_g the softmax of head g over keys
 * starts[b] .. col + t, out[row, h] = (sum_g talk[h, g] p_g) V_h * sigmoid(gate[row, g_off + h * dv ..]) (gate.ld 0: no gate),
 * V_h the values of head h's own kv head h / (H / G); caches as tnx_sink_attn's.  talk fp32 [H, H].  kv_chunk (a
 * multiple of 64 up to 320): keys of a work-group where T == 1.  ws: tnx_mixed_attn_ws_bytes.  tnx_mixed_attn_ok: whether a bf16 shape runs
 * on MFMA kernels; others, and fp32, run a plain kernel. */
typedef struct {
  int64_t B, T, S;
  int H, G, dk, dv, dkp, dvp;
  float scale;
  int dtype;
  const void* q;
  const void* kcache;
  const void* vcache;
  const float* talk;
  const int32_t* starts;
  const int32_t* col_ptr;
  int kv_chunk;
  float* ws;
  tnx_rows_src gate;
  int64_t g_off;
  void* out;
  int64_t out_ld;
  int out_frag;
} tnx_mixed_attn_desc;
int tnx_mixed_attn_ok(int64_t T, int64_t S, int H, int G, int dkp, int dvp);
size_t tnx_mixed_attn_ws_bytes(int64_t B, int64_t T, int64_t S, int H, int dvp, int kv_chunk);
int tnx_mixed_attn(void* stream, const tnx_mixed_attn_desc* d);

/* Matrix memory with exponential gates.  Per head, with i = cap tanh((gates[row, i_off + h] + bias_i[h]) / cap), f =
 * log sigmoid(cap tanh((gates[row, f_off + h] + bias_f[h]) / cap)) and the running maximum m (0 at a sequence's start):
 *   m' = max(f + m, i),  S' = e^(f + m - m') S + e^(i - m') k v^T,  n' the same with k alone,
 *   o[row, h * dv ..] = q_scale S'^T q / (max(|q_scale n'.q|, e^(-m')) + 1e-6).
 * y: q from q_off, k from k_off, v from v_off, head by head; gates: fp32 rows or planes.  state fp32 [B, H, dk, dv], sum
 * [B, H, dk] and top [B, H] are read unless col <= starts[b] and written back; o fp32 [B*T, o_ld].  ws:
 * tnx_memory_ws_bytes. */
typedef struct {
  int64_t B, T;
  int H, dk, dv;
  int dtype;
  float q_scale, cap;
  tnx_rows_src y;
  int64_t q_off, k_off, v_off;
  tnx_rows_src gates;
  int64_t i_off, f_off;
  const float* bias_i;
  const float* bias_f;
  const int32_t* starts;
  const int32_t* col_ptr;
  float* state;
  float* sum;
  float* top;
  float* o;
  int64_t o_ld;
  float* ws;
} tnx_memory_desc;
size_t tnx_memory_ws_bytes(int64_t B, int64_t T, int H, int dk, int dv);
int tnx_memory(void* stream, const tnx_memory_desc* d);

/* z <- cap * tanh(z / cap), n fp32 values in place. */
int tnx_soft_cap(void* stream, float* z, int64_t n, float cap);

/* Statistics and the whole-vocabulary draw of tnx_lmhead_logp over finished fp32 logits [M, V]
 * (any V); the fields mean what they mean there. */
typedef struct {
  int64_t M, V;
  const float* logits;
  float temperature;
  const int32_t* forbidden;
  int n_forbidden;
  const int32_t* targets;
  int32_t* best_id;
  float* best_logp;
  float* target_logp;
  float* lse;
  float* entropy;
  uint32_t draw_key0, draw_key1;
  int draw_rng_variant;
  const int32_t* draw_step_ptr;
  int32_t* draw_id;
  float* draw_logp;
} tnx_logits_desc;
int tnx_logits_stats(void* stream, const tnx_logits_desc* d);

#ifdef __cplusplus
}
#endif
#endif /* TUNIX_HIP_H_ */
