/* C ABI of libtriforce_latent.so: kernels of the latent-attention model family (models/modeling_befidra.py) for gfx950.
 *
 * Every entry point enqueues on `stream` and returns TF_OK, a TF_E* code (nothing launched) or a hipError_t.
 * dtype: 0 = bfloat16 operands with fp32 accumulation, 1 = everything in fp32.  "T" below is that element type.
 *
 * Padded sizes.  Every dimension that a matrix product contracts or tiles is padded to a multiple of 32 with zeros when the
 * weights are loaded; the kernels below only see padded sizes unless a parameter is called "real".  Names: H heads, N / R =
 * unrotated / rotated query-key size of a head, V = value size of a head, C = latent size (all padded), W = C + R = one
 * cached row: [latent C][rotated key R].
 *
 * Packed weights: a [n, k] matrix is stored as [n/16][k/32][64][8]: piece (g*16 + i) of a 16x32 tile holds
 * w[16a + i][32b + 8g .. +7] - one wavefront load per tile.
 */
#ifndef TRIFORCE_LATENT_H
#define TRIFORCE_LATENT_H
#include <stdint.h>
#ifndef TF_OK
#define TF_OK 0
#define TF_EINVAL (-22)
#define TF_ENOSPC (-28)
#define TF_ERANGE (-34)
#endif
#ifdef __cplusplus
extern "C" {
#endif

#define TFL_PAGE 64                 /* cache rows per page */

int tfl_abi_version(void);

/* Activation blocks: element (m, k) lives at m*ld + (k/8)*oct + k%8.  Row-major rows have oct = 8; decode keeps its norm output
 * and the output projection's input octet-major (ld = 8, oct = 8 * rows), where a 16-row operand is four contiguous runs. */

/* What a skinny GEMM does with its fp32 result (row m of x, output n of the group). */
enum {
    TFL_EPI_F32 = 0,                /* out_f[m*ld_f + n] = acc, n < n_real */
    TFL_EPI_IN = 1,                 /* n < n_raw: out_f[m*ld_f + n] = acc and ss[m*(n_raw/16) + n/16] = sum over the panel of
                                       acc^2, and for n < n_scaled out_t2 = acc * norm_w[n]
                                       (octet-major); else out_t(m, n - n_raw) = gelu_tanh(acc) */
    TFL_EPI_QUERY = 2,              /* acc *= 1 / sqrt(sum(ss_in[m][:ss_n]) / k_real + eps); heads of N + R outputs: out_t2[(m*H + h)*N + n] unrotated;
                                       out_t[(m*H + h)*(C + R) + C + n] rotated at pos[m] */
    TFL_EPI_LATENT = 3,             /* group h: out_t[(m*H + h)*(C + R) + n] = acc */
    TFL_EPI_GATED = 4,              /* group h: out_t(m, h*ppg*16 + n) = acc * sigmoid(gate[m*ld_gate + h*ppg*16 + n]) */
    TFL_EPI_RESIDUAL = 5,           /* out_f[m*ld_f + n] += acc; out_t(m, n) = the sum when out_t is given */
    TFL_EPI_TOKEN = 6               /* out_t[m*ld_t + n] = gelu_tanh(acc) * tok_table[ids[m]*ld_tok + n], n < n_real (0 behind) */
};
typedef struct TflGemm {
    const void* wp;                 /* packed weights, groups back to back */
    const void* x;
    const float* norm_w;            /* [n_scaled] */
    const float* ss_in;             /* [rows][ss_n]: the first ss_n panels' sums of squares, row stride ss_ld */
    void* out_t;
    void* out_t2;
    float* out_f;
    float* ss_out;
    const float* gate;
    const void* tok_table;
    const int64_t* ids;
    const int32_t* pos;
    const float* cos;               /* [max_pos][half] */
    const float* sin;
    /* key half of TFL_EPI_QUERY: extra workgroups normalise / rotate / store the cache row of every batch row */
    const float* kv_raw;            /* [rows] raw [latent C][rotated R] rows (NULL: none), row stride ld_kv */
    const float* kv_norm_w;         /* fp32 [C] */
    void* cache;                    /* [cache rows][C + R] */
    const int32_t* slot;            /* cache row per batch row; negative: nothing is stored */
    int64_t ld_x, x_oct, x_group, ld_t, t_oct, ld_f, ld_gate, ld_tok, ld_kv;
    int32_t rows, n, k, groups;     /* n = outputs per group, all groups alike */
    int32_t n_real, k_real, n_raw, n_scaled, ss_n, ss_ld;
    int32_t H, N, R, C, half, c_real, max_pos, cache_rows, vocab;
    float eps;
} TflGemm;

int tfl_gemm(const TflGemm* a, int dtype, int epilogue, void* stream);

/* x (fp32 residual) of one row per workgroup, in this order, each part optional:
 *   x = embed[ids]            (embed != NULL)
 *   x += y / rms(y) * y_w     (y != NULL; fp32 when y_f32, else T)
 *   x += step                 (step != NULL)
 *   h = x / rms(x) * norm_w   (T)
 * width_real elements carry data, rows have stride width (padded with zeros); h is an activation block (below). */
int tfl_finish(const void* embed, const int64_t* ids, int vocab, const void* y, int y_f32, int64_t ld_y, const float* y_w,
               const float* step, const float* norm_w, float* x, void* h, int64_t ld_h, int64_t h_oct, int rows, int width,
               int width_real, float eps, int dtype, void* stream);

/* x += d (T); xt = T(x)  (xt may be NULL). */
int tfl_residual(const void* d, float* x, void* xt, int64_t n, int dtype, void* stream);

/* out = gelu_tanh(s) * tok_table[ids[m]*ld_tok + n] for n < n_real, 0 behind. */
int tfl_token_gate(const void* s, int64_t ld_s, const void* tok_table, int64_t ld_tok, const int64_t* ids, int vocab, void* out,
                   int rows, int n, int n_real, int dtype, void* stream);

/* Prefill half of the input projection: y [rows][q + C + R + gate + up] (T) ->
 *   cq [rows][q] = y_q / rms * q_norm;  cache row slot[m] = latent / rms * kv_norm | rotated key;  ck [rows][C + R] the same
 *   row again (NULL: not wanted);  act [rows] at stride ld_act = gelu_tanh(up) (n_up = 0: none). */
int tfl_prepare(const void* y, int64_t ld_y, int q, int q_real, int C, int c_real, int R, int up_off, int n_up,
                const float* q_norm, const float* kv_norm, float eps, const float* cos, const float* sin, int half, int max_pos,
                const int32_t* pos, const int32_t* slot, void* cache, int cache_rows, void* cq, void* ck, void* act,
                int64_t ld_act, int rows, int dtype, void* stream);

/* dst[t] = cache[src[t]]: the cached rows of whole prefixes, packed. */
int tfl_gather_rows(const void* cache, int cache_rows, const int32_t* src, void* dst, int rows, int W, int dtype, void* stream);

/* Causal attention of packed new tokens over up-projected keys and values.
 *   q [tq][H*(N + R)] unrotated; the R part is rotated here at pos[token].
 *   kv [tk][H*N + H*V]: unrotated keys of all heads, then values;  ck [tk][C + R]: the rotated keys sit at column C.
 *   seq [nseq][4] int32: {first new token, new tokens, first key, keys}; new token j sees keys 0 .. keys - new + j.
 *   out [tq] at stride ld_out: o[h*V + d] * sigmoid(gate[token*ld_gate + h*V + d]) */
int tfl_attn_prefill(const void* q, const void* kv, const void* ck, const int32_t* seq, int nseq, int max_new, const int32_t* pos,
                     const float* cos, const float* sin, int half, int max_pos, const void* gate, int64_t ld_gate, void* out,
                     int64_t ld_out, int tq, int tk, int H, int N, int R, int V, int C, float scale, int dtype, void* stream);

/* One query token per sequence over the paged latent cache: q [rows][H][C + R] (keys are the cached rows themselves, values
 * their first C entries), len[row] keys (<= 0: output 0), page table [rows][table_ld].  out [rows][H][C] (T).
 * ws: tfl_attn_decode_ws_floats floats when nsplit > 1. */
int64_t tfl_attn_decode_ws_floats(int rows, int H, int C, int nsplit);
int tfl_attn_decode_pick_nsplit(int rows, int H, int max_len);
int tfl_attn_decode(const void* q, const void* cache, int n_pages, const int32_t* table, int table_ld, const int32_t* len,
                    void* out, float* ws, int64_t ws_floats, int rows, int H, int C, int R, float scale, int nsplit, int dtype,
                    void* stream);

/* Start of a decode step: pos = len; slot = table[len/64]*64 + len%64; klen = len + 1; len += 1.  Rows with len < 0 (or past
 * their table) stay idle: pos 0, slot -1, klen 0. */
int tfl_decode_prep(int32_t* len, const int32_t* table, int table_ld, int table_cols, int32_t* pos, int32_t* slot, int32_t* klen,
                    int rows, void* stream);

#ifdef __cplusplus
}
#endif
#endif
