// Layered models: kernels and launchers of the mechanisms a layer can be composed of (k_rows.hip, k_delta.hip,
// k_window.hip, k_latent.hip, k_gemm.hip).  Matrices are bf16 rows of `ld` elements (a multiple of 64, zero from K on); vectors,
// caches and recurrent state are fp32.
#pragma once

#include "l2h_internal.h"

struct LMat {
    uint16_t *w = nullptr;
    int64_t rows = 0;
    int K = 0, ld = 0;
    // tile image for the prompt pass (k_tiles.hip), or nullptr; elements of one matrix where several are stacked
    uint16_t *image = nullptr;
    int64_t image_stride = 0;
};
static inline int pad64(int64_t n) { return (int)((n + 63) / 64 * 64); }

static inline int pad4(int64_t n) { return (int)((n + 3) / 4 * 4); }

enum { LACT_GELU_ERF = 0, LACT_RELU2 = 1, LACT_GELU_TANH = 2, LACT_RELU = 3, LACT_SILU = 4 };
// how a router's logits become weights: a sigmoid each, on the expert's input, or the softmax over the chosen, on its output
enum { LROUTE_SIGMOID_IN = 0, LROUTE_SOFTMAX_OUT = 1 };

// ---- one token: matrix x vector with a fused prologue and epilogue (k_rows.hip) ---------------------------------
// prologues: what the vector in LDS is
//   RP_PLAIN    x
//   RP_NORM     rmsnorm(x) * normw; with y set, x first takes the pending update x += mult * rmsnorm(y) * yw, which
//               workgroup 0 also writes to x_out
//   RP_UP       as RP_NORM; the rows are those of the `top` experts with the largest z, `rows_each` rows each
//   RP_DOWN     x holds `top` vectors of K elements; every output row sums the chosen experts' rows
//   RP_HEADNORM x[h * hv + j] * rms over the head's hv elements (from partial sums of squares) * normw[j] * gate[...]
enum { RP_PLAIN = 0, RP_NORM = 1, RP_UP = 2, RP_DOWN = 3, RP_HEADNORM = 4 };
// epilogues: RE_STORE v; RE_RESID resid + mult * v; RE_ACT act(v); RE_UP act(score * v) or score * act(v) with the expert's score;
// RE_EMBED act(v) * the token's row of an embedding table; RE_GLU rows 2 i and 2 i + 1 give out[i] = act(v) * v', with the
// expert's score behind RP_UP; RE_STORE_GLU stores rows below glu_from and treats the others so, into out2
enum { RE_STORE = 0, RE_RESID = 1, RE_ACT = 2, RE_UP = 3, RE_EMBED = 4, RE_GLU = 5, RE_STORE_GLU = 6 };
struct RowsArgs {
    const uint16_t *w = nullptr;
    int ld = 0, K = 0;
    int64_t n_rows = 0;
    const float *x = nullptr;
    float *out = nullptr;
    float mult = 1.0f, eps = 0.0f;
    const float *normw = nullptr;
    const float *y = nullptr, *yw = nullptr;
    float *x_out = nullptr;
    const float *resid = nullptr;
    int act = 0;
    int64_t glu_from = 0;
    float *out2 = nullptr;
    const float *z = nullptr, *z_bias = nullptr;  // router logits
    int n_experts = 0, top = 0, route = 0;
    int64_t rows_each = 0;
    const float *ssq = nullptr, *gate = nullptr;  // RP_HEADNORM
    int hv = 0, n_split = 0;
    const uint16_t *emb = nullptr;  // RE_EMBED: element emb[token * emb_ld + row]
    int64_t emb_ld = 0;
    const DecodeCtl *ctl = nullptr;
    const int32_t *prompt = nullptr;
};
hipError_t k_rows(hipStream_t s, const RowsArgs &a, int pro, int epi, int n_cu);

// ---- many tokens: C[m][n] = sum_k X[m][k] W[n][k] (k_gemm.hip) ---------------------------------------------------
// activations are bf16 (prec 0) or fp32 (prec 1: fp32 products on the matrix cores); ldx a multiple of 64, zero from K on
enum {
    GE_STORE = 0,   // outf = v
    GE_RESID = 1,   // outf += mult * v
    GE_ACT = 2,     // outa = act(v)
    GE_UP = 3,      // outa = act(row_scale[m] * v), or row_scale[m] * act(v) without scale_in
    GE_EMBED = 4,   // outa = act(v) * embedding element
    GE_DECAY = 5,   // outf = -rate[n / hd] * softplus(v + bias[n]): the logarithm of a decay
    GE_SIGMOID = 6, // outf = sigmoid(v)
    GE_GLU = 7      // columns 2 i and 2 i + 1 give outa[i] = act(v) * v'; with row_scale as GE_UP, on both factors or on the result
};
struct GemmTile {  // a block of rows of a grouped product
    int32_t expert, row0, n;
};
struct GemmArgs {
    const uint16_t *w = nullptr;
    int64_t n_rows = 0;
    int ld = 0;
    const void *x = nullptr;
    int64_t ldx = 0;
    int M = 0;
    float *outf = nullptr;
    int64_t ldo = 0;
    void *outa = nullptr;  // activation-typed, columns up to acols (0: lda) are zeroed from the last result on
    int64_t lda = 0, acols = 0;
    int scale_in = 1;
    float mult = 1.0f;
    int act = 0;
    const float *row_scale = nullptr;
    const uint16_t *emb = nullptr;
    int64_t emb_ld = 0;
    const int32_t *tokens = nullptr;
    const float *rate = nullptr, *bias = nullptr;
    int hd = 1;
    // grouped form: tiles lists blocks of rows, each with its own matrix w + expert * expert_stride
    const GemmTile *tiles = nullptr;
    const int32_t *n_tiles = nullptr;
    int max_tiles = 0;
    int64_t expert_stride = 0;
    const int32_t *gather = nullptr;  // row of x for each row of the product
};
#define L_GEMM_TILE 128   // rows of a block for k_gemm ...
#define L_IMAGE_TILE 256  // ... and for k_tiles
hipError_t k_gemm(hipStream_t s, const GemmArgs &a, int prec, int epi);

// the same from a tile image (k_tiles.hip): GE_ACT, GE_GLU, and GE_UP / GE_GLU / GE_STORE in the grouped form; bf16 activations
hipError_t k_tiles(hipStream_t s, const GemmArgs &a, int epi);
int64_t k_tile_image_elems(int64_t rows, int ld);
hipError_t k_tile_image(hipStream_t s, const uint16_t *w, int ld, int64_t rows, int64_t n_mats, uint16_t *dst);
// outa[m][n] = act(v[m][n]) * embedding element, for products that the library has stored as fp32
hipError_t k_embed_rows(hipStream_t s, const float *v, int M, int N, int act, const uint16_t *emb, int64_t emb_ld,
                        const int32_t *tokens, void *outa, int64_t lda, int prec);

// rows of x (fp32, stride K): [x += mult * rmsnorm(y) * yw;] outa = rmsnorm(x) * w, or x itself with w == nullptr; with
// `gather`, row r of the result is row gather[r] of x
hipError_t k_norm_rows(hipStream_t s, float *x, int K, int M, const float *w, float eps, const float *y, const float *yw,
                       float mult, const int32_t *gather, void *outa, int64_t lda, int prec);

// ---- mixture of experts, many tokens (k_gemm.hip) ----------------------------------------------------------------
// z[M][ldz] (+ bias) -> choice[M][top], score[M][top]; then the grouping: slot_row / slot_scale per slot (slots of an expert are
// consecutive), slot_of[M][top], tiles
hipError_t k_route(hipStream_t s, const float *z, int64_t ldz, const float *bias, int M, int E, int top, int kind, int32_t *choice,
                   float *score);
hipError_t k_group(hipStream_t s, const int32_t *choice, const float *score, int M, int E, int top, int32_t *slot_row,
                   float *slot_scale, int32_t *slot_of, GemmTile *tiles, int32_t *n_tiles, int tile_rows);
// x[m] += mult * sum_k y[slot_of[m][k]]
hipError_t k_gather_add(hipStream_t s, float *x, const float *y, const int32_t *slot_of, int M, int top, int K, float mult);
// x[m] += a[m] + b, a or not
hipError_t k_stream_add(hipStream_t s, float *x, const float *a, const float *b, int M, int K);

// ---- gated delta rule with one decay per key channel (k_delta.hip) -----------------------------------------------
// The projected row of a token: q [G D] | k [G D] | v [H V] | beta logits [H] | decay factor [ra] | gate factor [rg].
struct DeltaShape {
    int H, G, D, V, taps, ra, rg;
    float eps;
    __host__ __device__ int channels() const { return 2 * G * D + H * V; }
    __host__ __device__ int off_b() const { return channels(); }
    __host__ __device__ int off_a() const { return channels() + H; }
    __host__ __device__ int off_g() const { return channels() + H + ra; }
    __host__ __device__ int n_in() const { return channels() + H + ra + rg; }
};
#define L_DELTA_COLS 32  // value columns per workgroup of the one-token kernel
static inline int delta_splits(int V) { return (V + L_DELTA_COLS - 1) / L_DELTA_COLS; }
struct DeltaWeights {
    const float *conv;  // [taps][channels], the current token's tap last
    const float *rate, *bias;  // [H], [H D]
    const uint16_t *a2, *g2;
    int lda2, ldg2;
};
// ring: [taps][channels], slot t % taps holds token t's projected channels; state: [H][D][V]
hipError_t k_delta_step(hipStream_t s, const DeltaShape &d, const DeltaWeights &w, const float *in, float *ring, float *state,
                        const DecodeCtl *ctl, float *o, float *ssq, float *gate);
// convolution, silu, unit vectors, beta: raw[M][ldr] -> qkv[M][channels], kq[M][G] (= k . q), beta[M][H], and the two low-rank
// factors as activations; qkv and the scan's o have room for a multiple of 16 rows
hipError_t k_delta_prepare(hipStream_t s, const DeltaShape &d, const float *conv, const float *raw, int64_t ldr, const float *ring,
                           int M, int pos0, float *qkv, float *kq, float *beta, void *fa, int64_t lfa, void *fg, int64_t lfg,
                           int prec);
// the recurrence over M tokens, logarithms of the decays in lg[M][H D]; o[M][H V]; then the ring takes the last tokens
hipError_t k_delta_scan(hipStream_t s, const DeltaShape &d, const float *qkv, const float *kq, const float *beta, const float *lg,
                        float *state, int M, int pos0, float *o);
// the same in chunks of 16 tokens on the matrix cores; rec: delta_walk_floats(d, M) floats of scratch
int64_t delta_walk_floats(const DeltaShape &d, int M);
hipError_t k_delta_walk(hipStream_t s, const DeltaShape &d, const float *qkv, const float *beta, const float *lg, float *state, int M,
                        int pos0, float *rec, float *o);
#define L_DELTA_WALK_MIN 24  // tokens from which the chunked form is used
hipError_t k_delta_ring(hipStream_t s, const DeltaShape &d, const float *raw, int64_t ldr, float *ring, int M, int pos0);
// outa[m][h V + j] = o * rms over the head * normw[j] * gate
hipError_t k_head_norm_rows(hipStream_t s, const float *o, const float *gate, const float *normw, int M, int H, int V, float eps,
                            void *outa, int64_t lda, int prec);

// ---- attention over a sliding window (k_window.hip) --------------------------------------------------------------
// The projected row of a token: q [H D] | k [G D] | v [G V] | gate logits [H].
struct WindowShape {
    int H, G, D, V, window, rot, gated, qk_norm;  // rot: rotated dimensions
    int rot_half;                                 // pairs i, i + rot / 2 instead of 2i, 2i+1
    float scale, eps;
    int seq_len;
    __host__ __device__ int Dp() const { return (D + 3) / 4 * 4; }  // key elements per cache row: kc[G][Dp / 4][seq_len][4]; vc[G][seq_len][V]
    __host__ __device__ int off_k() const { return H * D; }
    __host__ __device__ int off_v() const { return H * D + G * D; }
    __host__ __device__ int off_g() const { return H * D + G * D + G * V; }
    __host__ __device__ int n_in() const { return H * D + G * D + G * V + (gated ? H : 0); }
};
#define L_WIN_SPLIT 64  // keys per workgroup of the one-token kernel (a lane each)
static inline int window_splits(const WindowShape &w) { return (std::min(w.window, w.seq_len) + L_WIN_SPLIT - 1) / L_WIN_SPLIT; }
hipError_t k_window_step(hipStream_t s, const WindowShape &w, const float *freq, const float *in, float *kc, float *vc,
                         const DecodeCtl *ctl, float *part, float *out);
static inline int64_t window_part_floats(const WindowShape &w) { return (int64_t)w.H * window_splits(w) * (w.V + 2); }
// rotation + norm of q and k, cache append; q as fp32 [M][H D] (qf) or bf16 [M][H hs] (qb, zero beyond D)
hipError_t k_window_prepare(hipStream_t s, const WindowShape &w, const float *freq, const float *raw, int64_t ldr, float *kc,
                            float *vc, int M, int pos0, float *qf, uint16_t *qb, int hs);
// fp32 attention of M queries over the cache, output gate included
hipError_t k_window_rows(hipStream_t s, const WindowShape &w, const float *qf, const float *raw, int64_t ldr, const float *kc,
                         const float *vc, int M, int pos0, void *outa, int64_t lda, int prec);

// ---- attention over a cached latent (k_latent.hip) ---------------------------------------------------------------
// The projected row of a token: query latent [Q] | key/value latent [C] and rotated key part [R] | gates [H V], each part
// from a multiple of four on.  The cache holds a row of ld() floats per position: the normed latent, zeros up to Cp, the
// rotated part, zeros.  A head's key is [k_up c | rotated part], its value v_up c; one token's queries are taken through
// k_up^T instead, so that scores and values are formed on the cached rows, which all heads share, and v_up is applied to the
// result.  ukv: the rows of k_up (H D), then of v_up (H V), of C inputs.
struct LatentShape {
    int H, D, R, V, C, Q, rot, rot_half, gated;
    float scale, eps;
    int seq_len;
    __host__ __device__ int Cp() const { return (C + 15) / 16 * 16; }
    __host__ __device__ int Rp() const { return (R + 15) / 16 * 16; }
    __host__ __device__ int ld() const { return Cp() + Rp(); }
    __host__ __device__ int hq() const { return D + R; }
    __host__ __device__ int off_kv() const { return (Q + 3) / 4 * 4; }
    __host__ __device__ int off_g() const { return (off_kv() + C + R + 3) / 4 * 4; }
    __host__ __device__ int n_in() const { return (off_g() + (gated ? H * V : 0) + 3) / 4 * 4; }
};
#define L_LATENT_MAX_RANK 1024
#define L_LATENT_BLOCK 128  // tokens whose queries go through k_up^T at a time
#define L_LATENT_SMALL 16   // up to so many tokens of a prompt go that way, more through their heads' own keys and values
#define L_LATENT_SPLITS 128
// workgroups that share the keys of one block of 16 (token, head) columns
static inline int latent_splits(int64_t cols) {
    return (int)std::min<int64_t>(L_LATENT_SPLITS, std::max<int64_t>(1, 512 / ((cols + 15) / 16)));
}
static inline int64_t latent_part_floats(const LatentShape &w, int64_t cols) { return cols * latent_splits(cols) * (w.Cp() + 4); }
// raw[M][ldr] -> cache rows pos0 .., and the normed query latent as activations cq[M][lcq]
hipError_t k_latent_prepare(hipStream_t s, const LatentShape &w, const float *qnorm, const float *kvnorm, const float *freq,
                            const float *raw, int64_t ldr, float *cache, int M, int pos0, void *cq, int64_t lcq, int prec);
// q[M][H hq] -> qa[M H][ld]: rotated, the unrotated part through k_up^T.  With ctl the position is the decode step's and the
// token's own cache row is made from its projected row `in` by the same launch.
hipError_t k_latent_query(hipStream_t s, const LatentShape &w, const float *freq, const float *q, const uint16_t *ukv, int ldu,
                          float *qa, int M, int pos0, const DecodeCtl *ctl, const float *in, const float *kvnorm, float *cache);
// partial softmax sums of the cached rows, part: latent_part_floats(w, M H)
hipError_t k_latent_attend(hipStream_t s, const LatentShape &w, const float *qa, const float *cache, float *part, int M, int pos0,
                           const DecodeCtl *ctl);
// joins them, applies v_up and the gates raw[m][ldr]: outa[m][h V + e], columns H V .. cols - 1 zeroed
hipError_t k_latent_value(hipStream_t s, const LatentShape &w, const float *part, const uint16_t *ukv, int ldu, const float *raw,
                          int64_t ldr, int M, void *outa, int64_t lda, int64_t cols, int prec);
// for the matrix-core attention: rotated queries as bf16 [M][H hs], cached latents n rows from pos0 as activations [n][lda]
hipError_t k_latent_heads(hipStream_t s, const LatentShape &w, const float *freq, const float *q, uint16_t *qb, int hs, int M, int pos0);
hipError_t k_latent_rows(hipStream_t s, const LatentShape &w, const float *cache, int pos0, int n, uint16_t *outa, int64_t lda);
