/* C ABI of libomni_decoder.so: the kernels of decoder-only language models whose layers are described one by one (latent attention over a
 * paged cache of latents, windowed grouped attention over a paged cache of keys and values, a decaying linear recurrence and token shift with
 * per-sequence state, norms on outputs or behind sums, dense feed-forwards, a side embedding per layer).  Every entry launches on `stream`,
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
 *           post: x = (alpha * x_in[t] + y[t]) / sqrt(mean(..^2) + eps) * gain -- the norm behind the sum
 *   result  mu != NULL : h = x[t] + (x[t-1] - x[t]) * mu, x[t-1] of a batch's first token of a sequence from state[state_slot[row]]
 *                        (position 0: zeros);   use_final: h = final_gain * x / sqrt(mean(x^2) + eps);   else h = x
 *   a weight vector (elem [wp]) takes a gain's place where one is given: y_w for `gain`, final_w for `final_gain`
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
    float table_scale; /* ids: x = table_scale * table[ids[t]]; 0 stands for 1 */
    int post; float alpha; const void* y_w; const void* final_w;
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

/* Behind the joint projection proj fp32 [T, ld] (the sum of `slabs` such arrays) of a grouped attention layer, every head padded with zeros:
 *   [q heads * dp | k kv_heads * dp | v kv_heads * vp | gate logits heads * vp]        (kc == NULL: no k and v, another layer's are read;
 *                                                                                      gate == NULL: no gate logits)
 *   q[t]   = rotate(RMSnorm(all of q) * qw), k likewise with kw: the norm is over the whole projection (count heads * dim), weights padded as the heads
 *   rotate: dimensions i and i + rot_dims / 2 of a head turn by the angle whose (cos, sin) is rot[position][i]  (fp32 [rot_rows][rot_dims / 2][2])
 *   q elem [T, heads * dp]; keys and values into the cache, elem [blocks][kv_heads][block_size][dp or vp]; gate = sigmoid, elem [T, heads * vp]
 * rows >= *num_live (optional) leave the cache alone.                                                                                 */
typedef struct omni_qkv_write {
    const float* proj; int slabs; int64_t slab_stride; int ld, heads, kv_heads, dim, dp, vp;
    const void* qw; const void* kw; float eps; const float* rot; int rot_dims, rot_rows;
    void* q; void* kc; void* vc; void* gate;
    const int32_t* block_table; int bt_stride, block_size;
    const int32_t* row_of_tok; const int32_t* positions; const int32_t* num_live;
    int T, elem;
} omni_qkv_write;
int omni_qkv_write_run(const omni_qkv_write* a, void* stream);

/* out[t] = o[t] / sqrt(mean(o[t]^2) + eps) * w * sigmoid(gate[t]):  o fp32 [T, n] (count true values, the others zero), w elem [n].
 * slabs > 0: gate logits fp32 [T, ld] as the sum of `slabs` arrays; slabs = 0: elem [T, ld], already behind the sigmoid.
 * out elem [T, n], row-major or fragment-major (frag).                                                                                */
typedef struct omni_gated_norm {
    const float* o; const void* w; const void* gate; int slabs; int64_t slab_stride; int ld;
    int n, count; float eps; void* out; int frag, T, elem;
} omni_gated_norm;
int omni_gated_norm_run(const omni_gated_norm* a, void* stream);

/* out[t, h * n .. ] = x[t, h * k ..] . w[h]^T for every head h: bf16, w fragment-major [heads][n, k]; n % 16 == 0, k % 32 == 0.
 * out row-major [T, heads * n] or fragment-major (frag: heads * n % 32 == 0).                                                         */
int omni_head_gemm(const void* x, const void* w, void* out, int T, int heads, int n, int k, int frag, void* stream);

/* Activations of the products' epilogues.  OMNI_ACT_GELU_MUL: gelu_tanh(value) times the token's row of a table (omni_row_table)      */
#define OMNI_ACT_NONE 0
#define OMNI_ACT_XIELU 1
#define OMNI_ACT_RELU2 2
#define OMNI_ACT_GELU_MUL 3
/* value [m, n] is multiplied by table[ids[m] * ld + n] (table elem, n % 4 == 0 aligned; an id outside [0, rows): by zero)              */
typedef struct omni_row_table { const void* table; const int32_t* ids; int rows, ld; } omni_row_table;

/* fp32 GEMM, `batch` products: out[b] [M, N] = x[b] [M, K] . w[b]^T; element strides between products xb, wb, ob; act: OMNI_ACT_*      */
int omni_gemm_f32(const float* x, int ldx, int64_t xb, const float* w, int64_t wb, float* out, int ldo, int64_t ob, int M, int N, int K,
                  int batch, int act, float act_p, float act_n, void* stream);
/* ... with OMNI_ACT_GELU_MUL, one product                                                                                             */
int omni_gemm_f32_rows(const float* x, int ldx, const float* w, float* out, int ldo, int M, int N, int K, const omni_row_table* rt, void* stream);

/* Weight-streaming GEMM of up to 64 rows: x and w fragment-major bf16 (x [M, K] in whole 16-row tiles).
 *   kind 0: out fp32 [S][M, N], S = omni_gemm_stream_splits(M, N, K) partial sums over K (their sum is the product); `one`: S = 1
 *   kind 1: out bf16 [M, N], kind 2: bf16 xIELU(product), kind 3: bf16 relu(product)^2; row-major or fragment-major (out_frag)
 * omni_gemm_stream_rows: bf16 gelu_tanh(product) times the row table                                                                  */
#define OMNI_STREAM_MAX_SPLITS 4
int omni_gemm_stream(const void* x, const void* w, void* out, int M, int N, int K, int kind, int one, float act_p, float act_n, int out_frag, void* stream);
int omni_gemm_stream_rows(const void* x, const void* w, void* out, int M, int N, int K, const omni_row_table* rt, int out_frag, void* stream);
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

/* Causal grouped attention over a paged cache of keys and values (elem [blocks][kv_heads][block_size][dp or vp]); query head h reads key / value head
 * h / (heads / kv_heads):
 *   out[t, h] = gate[t, h] * sum_j w_j v_j,  w_j = exp(scale * q[t, h] . k_j) / (exp(sink[h]) + sum_j exp(..)),
 *   j <= positions[t], and positions[t] - j < window when window > 0
 * q elem [T, heads * dp]; gate (optional) and out elem [T, heads * vp], out row-major or fragment-major (frag); sink fp32 [heads] (optional: without
 * it the denominator is the sum alone).
 * Tokens [0, n_decode) are single-token sequences (workspace for the splits); the others are covered by `tiles` (int32 [n_tiles][2], device:
 * first flat row t * (heads / kv_heads) + r and row count <= tile_rows; one sequence each; every key / value head walks the same tiles).
 * max_keys bounds positions[t] + 1 of the decode tokens (split choice only).                                                          */
typedef struct omni_window_attn {
    const void* q; const void* kc; const void* vc; const void* gate; const float* sink; void* out; int frag;
    const int32_t* block_table; int bt_stride, block_size; const int32_t* row_of_tok; const int32_t* positions;
    const int32_t* tiles; int n_tiles, tile_rows;
    int T, n_decode, heads, kv_heads, dp, vp; float scale; int window, max_keys; float* workspace; int64_t workspace_bytes; int elem;
} omni_window_attn;
int omni_window_attn_run(const omni_window_attn* a, void* stream);
int64_t omni_window_attn_workspace_bytes(int n_decode, int heads, int vp);
int omni_window_attn_tile_rows(int dp, int vp);

/* Linear recurrence with one decay per head: S <- decay[h] * S + k v^T, out = S^T q, S fp32 [slots][heads][dp][vp] per sequence (state_slot[row];
 * a sequence's position 0 starts from zeros whatever the slot holds).
 * proj columns [q heads * dp | k heads * dp | v heads * vp | ...], heads padded with zeros:
 *   slabs > 0: fp32 [T, ld], the sum of `slabs` arrays, SiLU applied here;   slabs = 0: bf16 [T, ld], already behind it
 * out fp32 [T, heads * vp].
 *   runs    token by token: tokens [0, n_decode) one sequence each, then `runs` (int32 [n_runs][2], device: first token, count)
 *   chunks  (bf16 rows behind SiLU; dp, vp <= OMNI_REC_MAX_DIM): int32 [n_chunks][4] = first token, count <= OMNI_REC_CHUNK, index in its sequence's
 *           part of the batch, 0; segs int32 [n_segs][2] = first chunk, chunks.  chunk_states fp32 [n_chunks][heads][dp][vp]
 * rows >= *num_live (optional) leave state and out alone.                                                                             */
#define OMNI_REC_CHUNK 128
#define OMNI_REC_MAX_DIM 256
typedef struct omni_decay_rec {
    const void* proj; int slabs; int64_t slab_stride; int ld, heads, dp, vp;
    const float* decay; const float* log2_decay;
    float* state; const int32_t* state_slot; const int32_t* row_of_tok; const int32_t* positions; const int32_t* num_live;
    int n_decode; const int32_t* runs; int n_runs;
    const int32_t* chunks; int n_chunks; const int32_t* segs; int n_segs; float* chunk_states;
    float* out;
} omni_decay_rec;
int omni_decay_rec_run(const omni_decay_rec* a, void* stream);

/* The decode step's sampler: omni_sample_rows on rows < *num_live, ids into `ids` in place of the consumed ones, positions / seq_lens advanced */
int omni_sample_step(const float* logits, int ld, int B, int V, const omni_row_sampling* rows, uint8_t* seen, int32_t* steps, int32_t* ids,
                     int32_t* positions, int32_t* seq_lens, const int32_t* num_live, void* stream);

#ifdef __cplusplus
}
#endif
#endif
