/* C ABI of libomni_decoder.so: the kernels of decoder-only language models whose layers are described one by one (latent attention over a
 * paged cache of latents, token shift with per-sequence state, output norms, dense feed-forwards).  Every entry launches on `stream`,
 * allocates nothing, synchronises nothing (capturable) and returns OMNI_OK or an error with omni_last_error().
 *
 * The library also exports omni_gemm_tile and omni_sample / omni_sample_rows (omni_talker.h): same sources, linked without the talker.
 *
 * Conventions.  `elem`: 0 = bfloat16 (matrix operands, cache and activations bf16; sums, norms, scores, state fp32), 1 = fp32 throughout.
 * The residual stream x is fp32 [T, width] in both.  A batch is T tokens, sequence after sequence: row_of_tok[t] names the token's batch row
 * (one sequence), positions[t] its index in the sequence; a sequence's tokens of one batch are consecutive.  Widths are padded to
 * multiples of 32 with zero weights; norms take the unpadded width as their count.                                                    */
#ifndef OMNI_DECODER_H
#define OMNI_DECODER_H
#include "omni_talker.h"

#ifdef __cplusplus
extern "C" {
#endif

/* One pass over the residual stream between two sublayers:
 *   source  ids != NULL: x = table[ids[t]];  else x = x_in[t] + (y ? gain * y[t] / sqrt(mean(y[t]^2) + eps) : 0)      -> x_out (optional)
 *   result  mu != NULL : h = x[t] + (x[t-1] - x[t]) * mu, x[t-1] of a batch's first token of a sequence from state[state_slot[row]]
 *                        (position 0: zeros);   use_final: h = final_gain * x / sqrt(mean(x^2) + eps);   else h = x
 * h_out (optional) in `elem`, row-major [*, wp] or fragment-major (frag, bf16).  sel (optional): output i is token sel[i] (no mu, no x_out). */
typedef struct omni_stream_rows {
    const int32_t* ids; const void* table; int vocab;
    const float* x_in; const float* y; int y_slabs; int64_t y_stride; float gain, eps;     /* y = sum of y_slabs arrays y_stride elements apart (0, 1: one) */
    const void* mu; const float* state; const int32_t* state_slot; const int32_t* row_of_tok; const int32_t* positions;
    int use_final; float final_gain; const int32_t* sel;
    float* x_out; void* h_out; int frag;
    int rows;          /* tokens, or selected tokens */
    int width, wp;     /* true and padded width */
    int elem;
} omni_stream_rows;
int omni_stream_rows_run(const omni_stream_rows* a, void* stream);

/* Behind the joint down-projection proj fp32 [T, ld] (the sum of `slabs` such arrays) = [q latent (q_rank, padded to qp) | kv latent (kv_rank, padded to rp) | gate logits]:
 *   cq[t]  = RMSnorm(q part) * qw        elem [T, qp], row-major or fragment-major
 *   cache slot of (row, position)  = RMSnorm(kv part) * kw      elem [blocks, block_size, rp]
 *   gate[t, h] = sigmoid(gate logits)    fp32 [T, heads]        (gate != NULL)
 *   state[state_slot[row]] = x[t] for the last token of each sequence of the batch     (state != NULL)
 * rows >= *num_live (optional) leave cache and state alone.                                                                          */
typedef struct omni_latent_write {
    const float* proj; int slabs; int64_t slab_stride; int ld, q_rank, qp, kv_rank, rp, heads;
    const void* qw; const void* kw; float eps;
    void* cq; int frag; void* cache; float* gate;
    const int32_t* block_table; int bt_stride, block_size;
    const int32_t* row_of_tok; const int32_t* positions; const int32_t* num_live;
    const float* x; int wp; float* state; const int32_t* state_slot;
    int T, elem;
} omni_latent_write;
int omni_latent_write_run(const omni_latent_write* a, void* stream);

/* out[t, h * n .. ] = x[t, h * k ..] . w[h]^T for every head h: bf16, w fragment-major [heads][n, k]; n % 16 == 0, k % 32 == 0.
 * out row-major [T, heads * n] or fragment-major (frag: heads * n % 32 == 0).                                                         */
int omni_head_gemm(const void* x, const void* w, void* out, int T, int heads, int n, int k, int frag, void* stream);

/* fp32 GEMM, `batch` products: out[b] [M, N] = x[b] [M, K] . w[b]^T; element strides between products xb, wb, ob; act 0 none, 1 xIELU   */
int omni_gemm_f32(const float* x, int ldx, int64_t xb, const float* w, int64_t wb, float* out, int ldo, int64_t ob, int M, int N, int K,
                  int batch, int act, float act_p, float act_n, void* stream);

/* Weight-streaming GEMM of up to 64 rows: x and w fragment-major bf16 (x [M, K] in whole 16-row tiles).
 *   kind 0: out fp32 [S][M, N], S = omni_gemm_stream_splits(M, N, K) partial sums over K (their sum is the product); `one`: S = 1
 *   kind 1: out bf16 [M, N], kind 2: bf16 xIELU(product); row-major or fragment-major (out_frag)                                      */
#define OMNI_STREAM_MAX_SPLITS 4
int omni_gemm_stream(const void* x, const void* w, void* out, int M, int N, int K, int kind, int one, float act_p, float act_n, int out_frag, void* stream);
int omni_gemm_stream_splits(int M, int N, int K);

/* Causal attention over a paged cache of latents shared by all heads (keys and values are the same rp-wide rows):
 *   out[t, h] = gate[t, h] * sum_j softmax_j(scale * q[t, h] . c_j) c_j,   j <= positions[t],   q / out elem [T, heads, rp].
 * Tokens [0, n_decode) are single-token sequences (one work item per 16 heads and KV split; workspace for the splits); the others are
 * covered by `tiles` (int32 [n_tiles][2], device: first flat row t * heads + h and row count <= tile_rows; one sequence each;
 * tile_rows = omni_latent_attn_tile_rows(rp)).
 * max_keys bounds positions[t] + 1 of the decode tokens (split choice only).                                                        */
typedef struct omni_latent_attn {
    const void* q; const void* cache; const float* gate; void* out;
    const int32_t* block_table; int bt_stride, block_size; const int32_t* row_of_tok; const int32_t* positions;
    const int32_t* tiles; int n_tiles, tile_rows;
    int T, n_decode, heads, rp; float scale; int max_keys; float* workspace; int64_t workspace_bytes; int elem;
} omni_latent_attn;
int omni_latent_attn_run(const omni_latent_attn* a, void* stream);
int64_t omni_latent_attn_workspace_bytes(int n_decode, int heads, int rp);
int omni_latent_attn_tile_rows(int rp);
/* 1 when the matrix-core kernels take this padded latent width (else the plain kernel runs it) */
int omni_latent_attn_mfma(int rp);

/* The decode step's sampler: omni_sample_rows on rows < *num_live, ids into `ids` in place of the consumed ones, positions / seq_lens advanced */
int omni_sample_step(const float* logits, int ld, int B, int V, const omni_row_sampling* rows, uint8_t* seen, int32_t* steps, int32_t* ids,
                     int32_t* positions, int32_t* seq_lens, const int32_t* num_live, void* stream);

#ifdef __cplusplus
}
#endif
#endif
