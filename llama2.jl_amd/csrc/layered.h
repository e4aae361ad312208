// Layered models: kernels and launchers of the mechanisms a layer can be composed of (k_rows.hip, k_delta.hip,
// k_window.hip, k_gemm.hip).  Matrices are bf16 rows of `ld` elements (a multiple of 64, zero from K on); vectors,
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

enum { LACT_GELU_ERF = 0, LACT_RELU2 = 1, LACT_GELU_TANH = 2 };

// ---- one token: matrix x vector with a fused prologue and epilogue (k_rows.hip) ---------------------------------
// prologues: what the vector in LDS is
//   RP_PLAIN    x
//   RP_NORM     rmsnorm(x) * normw; with y set, x first takes the pending update x += mult * rmsnorm(y) * yw, which
//               workgroup 0 also writes to x_out
//   RP_UP       as RP_NORM; the rows are those of the `top` experts with the largest z, `rows_each` rows each
//   RP_DOWN     x holds `top` vectors of K elements; every output row sums the chosen experts' rows
//   RP_HEADNORM x[h * hv + j] * rms over the head's hv elements (from partial sums of squares) * normw[j] * gate[...]
enum { RP_PLAIN = 0, RP_NORM = 1, RP_UP = 2, RP_DOWN = 3, RP_HEADNORM = 4 };
// epilogues: RE_STORE v; RE_RESID resid + mult * v; RE_ACT act(v); RE_UP act(score * v) with the expert's score;
// RE_EMBED act(v) * the token's row of an embedding table
enum { RE_STORE = 0, RE_RESID = 1, RE_ACT = 2, RE_UP = 3, RE_EMBED = 4 };
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
    const float *z = nullptr;  // router logits
    int n_experts = 0, top = 0;
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
    GE_UP = 3,      // outa = act(row_scale[m] * v)
    GE_EMBED = 4,   // outa = act(v) * embedding element
    GE_DECAY = 5,   // outf = -rate[n / hd] * softplus(v + bias[n]): the logarithm of a decay
    GE_SIGMOID = 6  // outf = sigmoid(v)
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
    void *outa = nullptr;  // activation-typed, columns n_rows .. lda - 1 are zeroed
    int64_t lda = 0;
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

// the same from a tile image (k_tiles.hip): GE_ACT, and GE_UP / GE_STORE in the grouped form; bf16 activations
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
// z[M][E] -> choice[M][top], score[M][top]; then the grouping: slot_row / slot_scale per slot (slots of an expert are
// consecutive), slot_of[M][top], tiles
hipError_t k_route(hipStream_t s, const float *z, int M, int E, int top, int32_t *choice, float *score);
hipError_t k_group(hipStream_t s, const int32_t *choice, const float *score, int M, int E, int top, int32_t *slot_row,
                   float *slot_scale, int32_t *slot_of, GemmTile *tiles, int32_t *n_tiles, int tile_rows);
// x[m] += mult * sum_k y[slot_of[m][k]]
hipError_t k_gather_add(hipStream_t s, float *x, const float *y, const int32_t *slot_of, int M, int top, int K, float mult);

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
    int H, G, D, V, window, rot, gated, qk_norm;  // rot: rotated dimensions (pairs 2i, 2i+1)
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
