/*
 * msa_seq — C ABI of the gfx950 kernels behind the decoders of mixed layers: recurrences, latent attention, grouped-query
 * attention with chunk masks (libmsa_seq.so).
 *
 * Conventions are those of msa_amd.h (0 or a negative MSA_E* code, msa_last_error(), device pointers, everything
 * enqueued on `stream`, no allocation).  On top of them:
 *   - the rows of a step are the new tokens of `n_seq` sequences, concatenated; `msa_seq_batch` describes them.  What a
 *     sequence keeps between steps (last token, convolution inputs, recurrent states, latents) lives in caller-owned
 *     tensors indexed by the sequence's slot and is updated in place;
 *   - `dtype` is the activations' type; residual stream, norms, gates, decays, scores and states are fp32 always, and
 *     so are all small parameter vectors (norm weights, biases, taps, A_log, D, sinks);
 *   - strides are in elements.
 */
#ifndef MSA_SEQ_H
#define MSA_SEQ_H

#include "msa_amd.h"

#ifdef __cplusplus
extern "C" {
#endif

/* Host structure of device pointers: rows cu[s] .. cu[s + 1] - 1 belong to sequence s, row r to sequence row_seq[r];
 * slot[s] is the sequence's place in the state tensors, pos[s] the number of tokens it has already been fed.
 * `rows` = cu[n_seq], `max_rows` = the longest sequence of the step. */
typedef struct {
  const int32_t* cu;
  const int32_t* row_seq;
  const int32_t* slot;
  const int64_t* pos;
  int32_t n_seq, rows, max_rows, reserved;
} msa_seq_batch;

/* Dynamic-tanh norm of a row: tanh(alpha x) w + b.  A null `w` means no norm. */
typedef struct {
  const float* w;
  const float* b;
  float alpha;
  int32_t reserved;
} msa_dyn_tanh;

/* x_out = x_in + sigmoid(gate + gate_bias) * y  (fp32 stream; y == NULL: x_out is not written and may be NULL), then
 * h = norm(x_out), and with `shift`: h_shift[t] = h[t] + (h[t-1] - h[t]) * shift, the token before a sequence's first
 * row coming from prev[slot] ([slots, W] fp32, replaced by the last row's h; zeros for a new sequence).  x_out must
 * not alias x_in.  h may be NULL when only h_shift is wanted. */
int msa_seq_residual_norm(const float* x_in, const void* y, int64_t y_stride, const void* gate, int64_t gate_stride,
                          const float* gate_bias, float* x_out, int32_t dtype, int32_t W, const msa_dyn_tanh* norm,
                          void* h, const float* shift, float* prev, void* h_shift, const msa_seq_batch* batch, void* stream);

/* In place: the tanh form of gelu on columns [0, n) of `rows` rows. */
int msa_seq_gelu(void* y, int64_t y_stride, int32_t dtype, int32_t rows, int32_t n, void* stream);

/* out = cap * tanh(in / cap) (cap == 0: a copy), [rows, n] of `dtype` to fp32. */
int msa_seq_softcap(const void* in, int32_t dtype, int64_t n_elems, float cap, float* out, void* stream);

/* Operand of a projection of [x ; x0] that keeps the fp32 stream's precision in bf16 products: a row is
 * [bf16(x) | bf16(x - bf16(x)) | bf16(x0)] for MSA_BF16 and [x | x0] for MSA_F32. */
int msa_seq_join(const float* x, const float* x0, int32_t dtype, int32_t rows, int32_t W, void* out, void* stream);

/* Per-channel causal convolution over time + bias (or NULL) + silu of columns [0, C) of `in`; taps [C, K] (last column: the
 * current token), state [slots, K - 1, C] fp32 (the last K - 1 inputs, oldest first). */
int msa_seq_conv_silu(const void* in, int64_t in_stride, const float* taps, const float* bias, int32_t dtype, int32_t C,
                      int32_t K, float* state, void* out, int64_t out_stride, const msa_seq_batch* batch, void* stream);

/* Selective state-space recurrence, scalar decay per head, with the output gate:
 *   dt = softplus(dt_raw + dt_bias);  S <- exp(-exp(A_log) dt) S + dt B x^T;  v = (S^T C + D x) * silu(z)
 * xbc rows: [x: H P | B: G N | C: G N]; z [.., H P], dt_raw [.., H] with row strides; state [slots, H, N, P] fp32;
 * v [rows, H P] of `dtype`.  Token by token: the form for decoding, short portions and MSA_F32. */
int msa_seq_ssd_scan(const void* xbc, int64_t xbc_stride, const void* z, int64_t z_stride, const void* dt_raw, int64_t dt_stride,
                     const float* dt_bias, const float* A_log, const float* D, int32_t dtype, int32_t H, int32_t P, int32_t N,
                     int32_t G, float* state, void* v, const msa_seq_batch* batch, void* stream);
/* The same recurrence for long bf16 portions, in chunks of 64 or 128 tokens on the matrix cores: chunk states, their
 * recurrence, chunk outputs.  N a multiple of 8 up to 256, P a multiple of 8. */
size_t msa_seq_ssd_chunked_workspace_bytes(int32_t max_rows, int32_t n_seq, int32_t H, int32_t P, int32_t N);
int msa_seq_ssd_chunked(const void* xbc, int64_t xbc_stride, const void* z, int64_t z_stride, const void* dt_raw, int64_t dt_stride,
                        const float* dt_bias, const float* A_log, const float* D, int32_t dtype, int32_t H, int32_t P,
                        int32_t N, int32_t G, float* state, void* v, const msa_seq_batch* batch, void* workspace,
                        size_t workspace_bytes, void* stream);

/* RMS norm of n columns in `parts` equal parts, times w: [rows, n] dense of `dtype`. */
int msa_seq_group_rmsnorm(const void* v, int32_t dtype, int32_t rows, int32_t n, int32_t parts, const float* w, float eps,
                          void* out, void* stream);

/* Minimal gated recurrence, element by element: z = sigmoid(z_raw + z_bias), u = u_raw + u_bias, candidate u + 1/2 for
 * u >= 0 and sigmoid(u) below, S <- (1 - z) S + z candidate, out = S * silu(g).  `zug` rows hold groups of 48 columns
 * [16 z | 16 u | 16 g] of the same 16 channels (n padded to a multiple of 16); state [slots, n] fp32.  Workspace: msa_seq_min_gru_workspace_bytes (0 when no sequence has more than one chunk). */
size_t msa_seq_min_gru_workspace_bytes(int32_t rows, int32_t n_seq, int32_t max_rows, int32_t n);
int msa_seq_min_gru(const void* zug, int64_t zug_stride, const float* z_bias, const float* u_bias, int32_t dtype, int32_t n,
                    float* state, void* out, const msa_seq_batch* batch, void* workspace, size_t workspace_bytes, void* stream);

/* c = rms_norm(in) * w of `rank` columns, written to the latent cache [slots, Lcap, rank] (dtype) at the rows'
 * positions.  Rows past the capacity are an error of the caller: they are not written. */
int msa_seq_latent_append(const void* in, int64_t in_stride, const float* w, float eps, int32_t dtype, int32_t rank,
                          void* cache, int64_t Lcap, const msa_seq_batch* batch, void* stream);

/* Causal attention over cached latents: q [rows, H, rank] (queries already multiplied by their heads' key matrices),
 * ctx[r, h] = sum_j p_j c_j with p = exp(s_j) / (exp(sink_h) + sum exp(s_j)), s = q . c * scale, j <= the row's position.
 * msa_seq_latent_attn: any rank, one workgroup per (row, head).  msa_seq_latent_decode: bf16, rank a multiple of 8 up
 * to 512, keys split over workgroups and all heads of a row from one pass over the latents; max_keys bounds
 * pos + rows of every sequence. */
int msa_seq_latent_attn(const void* q, const void* cache, int64_t Lcap, const float* sink, float scale, int32_t dtype,
                        int32_t H, int32_t rank, void* ctx, const msa_seq_batch* batch, void* stream);
size_t msa_seq_latent_decode_workspace_bytes(int32_t rows, int32_t H, int32_t rank, int64_t max_keys);
int msa_seq_latent_decode(const void* q, const void* cache, int64_t Lcap, const float* sink, float scale, int32_t dtype,
                          int32_t H, int32_t rank, int64_t max_keys, void* ctx, const msa_seq_batch* batch, void* workspace,
                          size_t workspace_bytes, void* stream);

/* Causal attention of a block of query rows over per-head keys and values (bf16): q [rows, H, D] with a row stride, and
 * for sequence s keys k[kv_off[s] + j, h G / H, :D], values v[kv_off[s] + j, h G / H, :E], j < pos[s] + its rows, with row
 * strides.  `chunk` > 0: position i sees j >= i / chunk * chunk only.  `sink` [H] (or NULL) enters the denominators as in
 * msa_seq_latent_attn; `gate` [rows, H] (or NULL): head outputs times sigmoid(gate).  D and E multiples of 8 up to 256.
 * out [rows, H, E] dense. */
int msa_seq_flash(const void* q, int64_t q_stride, const void* k, int64_t k_stride, const void* v, int64_t v_stride,
                  const int64_t* kv_off, const float* sink, float scale, int32_t dtype, int32_t H, int32_t G, int32_t D, int32_t E,
                  int32_t chunk, const void* gate, int64_t gate_stride, void* out, const msa_seq_batch* batch, void* stream);

/* What stands between the projections of a grouped-query attention layer and its scores: RMS norm of every query and key
 * head (q_norm / k_norm [D]), rotation of the first 2 n_pairs dimensions (pair i: dimensions i and i + n_pairs, angle
 * position * freqs[i] radians, freqs fp64 [n_pairs]), keys and values to the caches k_cache [slots, Lcap, G, D] and
 * v_cache [slots, Lcap, G, E].  q_out [rows, H, D] dense.  k == NULL: queries only.  D up to 512. */
typedef struct {
  const void* q;
  const void* k;
  const void* v;
  int64_t q_stride, k_stride, v_stride;
  const float* q_norm;
  const float* k_norm;
  const double* freqs;
  void* q_out;
  void* k_cache;
  void* v_cache;
  int64_t Lcap;
  int32_t H, G, D, E, n_pairs;
  float eps;
} msa_qk_rope_args;
int msa_seq_qk_rope_append(const msa_qk_rope_args* args, int32_t dtype, const msa_seq_batch* batch, void* stream);

/* Causal attention of prepared queries q [rows, H, D] over those caches, with the chunk mask and the output gate of
 * msa_seq_flash; out [rows, H, E] dense.
 * msa_seq_kv_attn: any sizes and type, one workgroup per (row, head).  msa_seq_kv_decode: bf16, D and E multiples of 8 up
 * to 256; the keys of a row are split over wavefronts and workgroups, the query heads of a key head share one pass;
 * max_keys bounds pos + rows of every sequence. */
typedef struct {
  const void* q;
  const void* k_cache;
  const void* v_cache;
  const void* gate;
  void* out;
  int64_t Lcap, gate_stride, max_keys;
  int32_t H, G, D, E, chunk;
  float scale;
} msa_kv_attn_args;
int msa_seq_kv_attn(const msa_kv_attn_args* args, int32_t dtype, const msa_seq_batch* batch, void* stream);
size_t msa_seq_kv_decode_workspace_bytes(const msa_kv_attn_args* args, int32_t rows);
int msa_seq_kv_decode(const msa_kv_attn_args* args, const msa_seq_batch* batch, void* workspace, size_t workspace_bytes, void* stream);

/* Delta rule with a decay per key channel.  qkv rows [q: G D | k: G D | v: H E] (after convolution and silu); per head h, with
 * q and k those of key head h G / H as unit vectors (1e-6 under the root), q times D^-1/2:
 *   S <- exp(-exp(A_log) softplus(a + dt_bias)) S  (row by row of S [D, E]);  u = sigmoid(b) (v - S^T k);  S <- S + k u^T;  o = S^T q
 *   out = o / rms(o) * norm * sigmoid(gate)
 * a [rows, H D], b [rows, H], gate [rows, H E] with row strides; dt_bias [H D], norm [E]; state [slots, H, D, E] fp32;
 * out [rows, H E] of `dtype`.
 * msa_seq_delta_scan: token by token, D up to 512.  msa_seq_delta_chunked: long bf16 portions in chunks of 64 tokens on the
 * matrix cores, D and E multiples of 8, D up to 128. */
typedef struct {
  const void* qkv;
  const void* a;
  const void* b;
  const void* gate;
  int64_t qkv_stride, a_stride, b_stride, gate_stride;
  const float* A_log;
  const float* dt_bias;
  const float* norm;
  float* state;
  void* out;
  int32_t H, G, D, E;
  float eps;
  int32_t reserved;
} msa_delta_args;
int msa_seq_delta_scan(const msa_delta_args* args, int32_t dtype, const msa_seq_batch* batch, void* stream);
size_t msa_seq_delta_chunked_workspace_bytes(const msa_delta_args* args, int32_t max_rows, int32_t n_seq);
int msa_seq_delta_chunked(const msa_delta_args* args, const msa_seq_batch* batch, void* workspace, size_t workspace_bytes, void* stream);

/* In place on [rows, H, E] dense: o / rms(o) * norm [E] * sigmoid(gate). */
int msa_seq_head_norm_gate(void* o, const void* gate, int64_t gate_stride, const float* norm, float eps, int32_t dtype, int32_t rows,
                           int32_t H, int32_t E, void* stream);

/* x_out = x_in + rms_norm(y) * w (fp32 stream, may alias; y == NULL: x_in itself, nothing written), and h = x_out, or
 * rms_norm(x_out) * next_w when given, in `dtype` (NULL: not wanted).  [rows, W]. */
int msa_seq_rms_residual(const float* x_in, const void* y, int64_t y_stride, const float* w, float eps, float* x_out,
                         const float* next_w, void* h, int32_t dtype, int32_t rows, int32_t W, void* stream);

/* Gated linear unit with clamped inputs on rows of n (gate, up) pairs: with g = min(gate, limit), u = clamp(up, -limit,
 * limit), out = g sigmoid(alpha g) (u + shift); out [rows, n] dense. */
int msa_seq_clamped_glu(const void* in, int64_t in_stride, int32_t dtype, int32_t rows, int32_t n, float limit, float alpha,
                        float shift, void* out, void* stream);

/* Weight-streaming linear for the M <= 16 rows of a decode step (bf16 operands, fp32 sums): row m of the product is
 * W[n, :K] . x[m, :K] for n < N, in `groups` groups: group g takes weight rows g N .. and columns x + g K.
 * Rows n >= n_b of the weights read x_b instead of x (n_b = N: all read x).  Epilogues (fields unused by one are ignored):
 *   MSA_ROWS_PLAIN    out[m, g N + n] = act(product): bf16, columns [0, gelu_n) through gelu
 *   MSA_ROWS_F32      out fp32, softcapped when cap > 0, plus add[n] when given
 *   MSA_ROWS_RESIDUAL x_out = x_in + sigmoid(gate + gate_bias) * product (fp32, may alias), then norm, h and the token shift
 *                     as msa_seq_residual_norm does (one row per sequence)
 *   MSA_ROWS_MAMBA    columns [z: conv_lo | conv input: conv_n | dt | (x_b rows)]: the conv columns leave through the
 *                     causal convolution + silu with their state updated, the others as they are
 *   MSA_ROWS_GLU      weight rows in (gate, up) pairs: out[m, n / 2] = the clamped gated unit of msa_seq_clamped_glu
 *   MSA_ROWS_GRU      weights in 48-row groups [16 z | 16 u | 16 g] of the same 16 channels (x_b rows behind them plain): the
 *                     recurrence of msa_seq_min_gru, out2[m, channel]
 */
#define MSA_ROWS_PLAIN 0
#define MSA_ROWS_F32 1
#define MSA_ROWS_RESIDUAL 2
#define MSA_ROWS_MAMBA 3
#define MSA_ROWS_GRU 4
#define MSA_ROWS_GLU 5
typedef struct {
  const void* x;
  const void* x_b;
  const void* w;
  void* out;
  int64_t x_stride, x_b_stride, out_stride;
  int32_t M, N, K, groups, n_b, gelu_n;
  float cap;
  int32_t reserved;
  const float* add;
  /* residual */
  const float* x_in;
  float* x_out;
  const void* gate;
  int64_t gate_stride;
  const float* gate_bias;
  msa_dyn_tanh norm;
  void* h;
  const float* shift;
  float* prev;
  void* h_shift;
  /* mamba */
  const float* taps;
  const float* conv_bias;
  float* conv_state;
  int32_t conv_lo, conv_n, conv_k, reserved2;
  /* gru */
  const float* z_bias;
  const float* u_bias;
  float* gru_state;
  void* out2;
  int32_t gru_n, reserved3;
  const int32_t* slot;
  /* clamped gated unit */
  float glu_limit, glu_alpha, glu_shift;
  int32_t reserved4;
} msa_rows_args;
int msa_rows_linear(const msa_rows_args* args, int32_t epilogue, void* stream);

#ifdef __cplusplus
}
#endif
#endif /* MSA_SEQ_H */
