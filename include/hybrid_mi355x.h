/*
 * hybrid_mi355x.h - C ABI of the MI355X (gfx950) kernels for decoders with unquantised weights whose
 * layers mix gated linear attention and latent attention.
 *
 * Plain pointers and sizes only; every tensor pointer is a DEVICE pointer, `stream` a hipStream_t.
 * All entry points are asynchronous and stream ordered, never synchronise, never allocate and never
 * retain pointers, and are safe under HIP-graph capture.  Argument errors are detected on the host
 * before any device work.  Return value: 0 or an hyb_status code.
 *
 * Storage: `dtype` says how weights, activations and cached latents are held (bf16 or fp32; fp32
 * products run on the fp32 matrix instructions).  The residual stream, norm weights, biases, scores,
 * decays and recurrent states are always fp32.
 *
 * Padding: inner dimensions are multiples of 64 and head dimensions multiples of 16 or 32; the caller
 * pads weights with zeros, so that pad columns of every product are zero.  *_true arguments give
 * the size that counts in a mean.
 *
 * Live rows: a launch is laid out for R (or M) rows, of which *n_dev (NULL: all) are live; the others
 * are neither read as input nor written.  len_dev: tokens in the cache before this pass.
 */
#ifndef HYBRID_MI355X_H
#define HYBRID_MI355X_H

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

typedef void* hyb_stream_t; /* hipStream_t */

enum hyb_status {
  HYB_OK = 0,
  HYB_ERR_NULL = 1,
  HYB_ERR_SHAPE = 2,
  HYB_ERR_ALIGN = 3,
  HYB_ERR_UNSUPPORTED = 4,
  HYB_ERR_WORKSPACE = 5,
  HYB_ERR_HIP = 6
};
enum hyb_dtype { HYB_BF16 = 0, HYB_F32 = 1 };

#define HYB_GLA_CHUNK 64 /* rows per chunk of the linear-attention prompt form */

const char* hyb_status_string(int status);
int hyb_abi_version(void);

/* h[r] = table[tokens[r]] * scale + pos_table[*len_dev + r] (pos_table may be NULL); h fp32 [R][D]. */
int hyb_embed(int dtype, const int32_t* tokens, const void* table, float scale, const void* pos_table, int max_positions,
              const int32_t* len_dev, const int32_t* n_dev, float* h, int R, int D, int V, hyb_stream_t stream);

/* out[r] = x[row] / sqrt(mean(x[row]^2) + eps) * w, row = rows ? rows[r] : r; x fp32 [.][D], the mean
 * over d_true columns (the others are zero), w fp32 [D]. */
int hyb_norm_rows(int dtype, const float* x, const int32_t* rows, const float* w, float eps, void* out, const int32_t* n_dev,
                  int R, int D, int d_true, hyb_stream_t stream);

/* out = epilogue(x W^T + bias).  x [M][ldx], W [N][K], both of `dtype`.
 *   HYB_OUT_T           out of `dtype` [M][ldo]
 *   HYB_OUT_F32         out fp32
 *   HYB_OUT_ADD_F32     out fp32 += (the residual stream)
 *   HYB_OUT_RELU2       out of `dtype` = max(y, 0)^2
 *   HYB_OUT_TRANSPOSED  out of `dtype` [N][ldo], out[n][m]; ldo % 128 == 0, no bias
 * norm_w != NULL: x is the fp32 residual stream and is RMS-normalised first (hyb_norm_rows; M <= 4).
 * len_dev != NULL: x is a token-indexed buffer (a cache) and row m of the product is its row
 * max(0, *len_dev - back) + m, up to row *len_dev + *n_dev - 1.
 * Forms: ROWS (vector ALU, M <= 4), SKINNY (16-row weight tiles, M <= 64), GEMM (LDS-tiled); form < 0
 * picks by hyb_dense_form.  N % 16 == 0, K % 64 == 0. */
enum hyb_epilogue { HYB_OUT_T = 0, HYB_OUT_F32 = 1, HYB_OUT_ADD_F32 = 2, HYB_OUT_RELU2 = 3, HYB_OUT_TRANSPOSED = 4 };
enum hyb_form { HYB_FORM_ROWS = 0, HYB_FORM_SKINNY = 1, HYB_FORM_GEMM = 2 };
typedef struct {
  const void* x;
  const void* w;
  const float* bias;
  void* out;
  const int32_t* n_dev;
  const int32_t* len_dev;
  const float* norm_w;
  long ldx, ldo;
  int dtype, M, N, K, epilogue, back, norm_d, form;
  float eps;
} hyb_dense_args;
int hyb_dense_form(int dtype, int M, int K, int norm, int transposed);
int hyb_dense(const hyb_dense_args* args, hyb_stream_t stream);

/* Gated linear attention of one layer over R rows: S <- diag(sigmoid(z)^(1/tau)) S + k v^T,
 * o = S^T (q qscale), out = o / rms(o) * norm_w * silu(gate), per head.
 * x [R][ldx] holds the fused projection: q and k (H x dkp), v and gate (H x dvp) at column offsets
 * off_*; state fp32 [H][dkp][dvp], updated.
 *   hyb_gla_step:   few rows; the decay's second factor is applied inside (a1 part of x at off_a,
 *                   rp columns; a2 [H dkp][rp], a2_bias fp32);
 *   hyb_gla_chunks: R % 64 == 0 rows; z fp32 [R][H dkp] (with bias) is given and overwritten. */
typedef struct {
  const void* x;
  const void* a2;
  const float* a2_bias;
  float* z;
  const float* norm_w;
  float* state;
  void* out;
  const int32_t* n_dev;
  void* workspace;
  size_t workspace_bytes;
  long ldx, ldo;
  int dtype, R, H, dkp, dvp, rp, dv_true, off_q, off_k, off_v, off_g, off_a;
  float qscale, tau, eps;
} hyb_gla_args;
int hyb_gla_step(const hyb_gla_args* args, hyb_stream_t stream);
size_t hyb_gla_chunk_workspace_bytes(int R, int H, int dkp, int dvp);
int hyb_gla_chunks(const hyb_gla_args* args, hyb_stream_t stream);

/* cache[*len_dev + r] = x[r] / sqrt(mean(x[r]^2) + eps) * w; cache [cap][rank] of `dtype`. */
int hyb_latent_append(int dtype, const void* x, long ldx, const float* w, float eps, void* cache, long cap,
                      const int32_t* len_dev, const int32_t* n_dev, int R, int rank, int rank_true, hyb_stream_t stream);

/* Latent attention of few rows (R <= 64) with absorbed key projection: position i = *len_dev + r sees the cached
 * rows j with 0 <= i - j < window.  append [R][ldappend]: the new rows before their norm, normed and appended
 * first as by hyb_latent_append; NULL where they are in the cache already.  q [R][ldq] (H x dp), uk [H dp][rank],
 * uv [H dvp][rank], gate [R][ldg] (H x dvp): out[r] = (softmax(scale q.k) v) * sigmoid(gate). */
typedef struct {
  const void* q;
  void* cache;
  const void* uk;
  const void* uv;
  const void* gate;
  void* out;
  const int32_t* len_dev;
  const int32_t* n_dev;
  void* workspace;
  size_t workspace_bytes;
  const void* append;
  const float* append_norm;
  long ldq, ldg, ldo, cap, ldappend;
  int dtype, R, H, dp, dvp, rank, window, rank_true;
  float scale, eps;
} hyb_latent_decode_args;
int hyb_latent_rank_supported(int rank);
size_t hyb_latent_decode_workspace_bytes(int R, int H, int rank, int window, long cap);
int hyb_latent_decode(const hyb_latent_decode_args* args, hyb_stream_t stream);

/* The same over projected keys and values (a prompt portion): k [S][ldk] (H x dp), vt [H dvp][ldv]
 * (transposed), row s = position max(0, *len_dev - back) + s, back >= min(window - 1, *len_dev).
 * dp % 32 == 0, dvp % 16 == 0, both <= 256; ldv % 64 == 0 and k has ldv rows, all finite. */
typedef struct {
  const void* q;
  const void* k;
  const void* vt;
  const void* gate;
  void* out;
  const int32_t* len_dev;
  const int32_t* n_dev;
  long ldq, ldk, ldv, ldg, ldo;
  int dtype, R, H, dp, dvp, window, back;
  float scale;
} hyb_window_args;
int hyb_window_attention(const hyb_window_args* args, hyb_stream_t stream);

/* Row argmax of fp32 logits [R][ld], lowest index among equal maxima. */
size_t hyb_argmax_workspace_bytes(int R);
int hyb_argmax_rows_f32(const float* logits, long ld, int R, int V, int32_t* out, void* workspace, size_t workspace_bytes,
                        hyb_stream_t stream);

/* Loop state on the device: *next = *token, out[*count] = *token (while *count < max_out), *count += 1. */
int hyb_token_advance(const int32_t* token, int32_t* next, int32_t* out, int32_t* count, int max_out, hyb_stream_t stream);
/* *len_dev = min(*len_dev + *n_dev, capacity) */
int hyb_advance_len(int32_t* len_dev, const int32_t* n_dev, int capacity, hyb_stream_t stream);

#ifdef __cplusplus
}
#endif
#endif /* HYBRID_MI355X_H */
