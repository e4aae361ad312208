// Attention over a cached latent: the cache holds one normed latent and one rotated key part per position, which all heads
// share.  For few tokens the queries are taken through k_up^T, so that scores and value sums are formed on the cached rows
// themselves (fp32 matrix cores), and v_up is applied once per token.  Everything is fp32; matrices are bf16 rows.
#include "layered_dev.h"

typedef float lat_f32x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float4 lat_zero4() { return make_float4(0.f, 0.f, 0.f, 0.f); }

// ---------------------------------------------------------------------------------------------------------------
// a position's cache row, by one workgroup of 256: src holds the projected [C | R] elements (C <= 1024), red four floats
// ---------------------------------------------------------------------------------------------------------------
__device__ __forceinline__ void lat_cache_row(const LatentShape &w, const float *kvnorm, const float *freq, const float *src, int pos,
                                              float *row, float *red) {
    constexpr int N = L_LATENT_MAX_RANK / 256;
    const int t = threadIdx.x, lane = t & 63, Cp = w.Cp();
    float v[N], g[N], ss = 0.0f;
#pragma unroll
    for (int u = 0; u < N; u++) {
        const int i = min(t + 256 * u, w.C - 1);
        v[u] = src[i];
        g[u] = kvnorm[i];
    }
    if (t >= 192) {
        l_rotate_norm(src + w.C, row + Cp, w.R, w.rot, w.rot_half, freq, pos, 0, 0.0f, lane);
        for (int i = w.R + lane; i < w.Rp(); i += 64) row[Cp + i] = 0.0f;
    }
#pragma unroll
    for (int u = 0; u < N; u++)
        if (t + 256 * u < w.C) ss = fmaf(v[u], v[u], ss);
    const float r = 1.0f / sqrtf(l_block_sum(ss, red) / (float)w.C + w.eps);
#pragma unroll
    for (int u = 0; u < N; u++) {
        const int i = t + 256 * u;
        if (i < Cp) row[i] = i < w.C ? v[u] * r * g[u] : 0.0f;
    }
}

// many tokens: one workgroup each
template <int PREC>
__global__ __launch_bounds__(256) void latent_prepare_kernel(LatentShape w, const float *qnorm, const float *kvnorm, const float *freq,
                                                             const float *raw, int64_t ldr, float *cache, int pos0, void *cq, int64_t lcq) {
    __shared__ float s_red[4];
    const int64_t m = blockIdx.x;
    const int t = threadIdx.x, pos = pos0 + (int)m;
    const float *src = raw + m * ldr;
    // (lcq is a multiple of 64; rows of raw and their part of Q elements begin on a multiple of four and are padded to one)
    constexpr int N = 2;  // quads a thread keeps
    float4 v[N];
    float ss = 0.0f;
    auto quad = [&](int i) { return i < w.Q ? *(const float4 *)(src + i) : lat_zero4(); };
    auto add = [&](float4 a, int i) {
        const float x[4] = {a.x, a.y, a.z, a.w};
#pragma unroll
        for (int e = 0; e < 4; e++)
            if (i + e < w.Q) ss = fmaf(x[e], x[e], ss);
    };
#pragma unroll
    for (int u = 0; u < N; u++) v[u] = quad(4 * (t + 256 * u));
#pragma unroll
    for (int u = 0; u < N; u++) add(v[u], 4 * (t + 256 * u));
    for (int i = 4 * (t + 256 * N); i < w.Q; i += 1024) add(quad(i), i);
    lat_cache_row(w, kvnorm, freq, src + w.off_kv(), pos, cache + (int64_t)pos * w.ld(), s_red);
    const float rq = 1.0f / sqrtf(l_block_sum(ss, s_red) / (float)w.Q + w.eps);
    auto put = [&](float4 a, int i) {
        const float x[4] = {a.x, a.y, a.z, a.w};
        float o[4];
#pragma unroll
        for (int e = 0; e < 4; e++) o[e] = i + e < w.Q ? x[e] * rq * qnorm[i + e] : 0.0f;
        if (PREC)
            *(float4 *)((float *)cq + m * lcq + i) = make_float4(o[0], o[1], o[2], o[3]);
        else
            *(uint2 *)((uint16_t *)cq + m * lcq + i) = make_uint2(l_pack_bf16(o[0], o[1]), l_pack_bf16(o[2], o[3]));
    };
#pragma unroll
    for (int u = 0; u < N; u++)
        if (4 * (t + 256 * u) < lcq) put(v[u], 4 * (t + 256 * u));
    for (int i = 4 * (t + 256 * N); i < lcq; i += 1024) put(quad(i), i);
}
hipError_t k_latent_prepare(hipStream_t s, const LatentShape &w, const float *qnorm, const float *kvnorm, const float *freq,
                            const float *raw, int64_t ldr, float *cache, int M, int pos0, void *cq, int64_t lcq, int prec) {
    if (M < 1 || pos0 < 0 || pos0 + M > w.seq_len || ldr < w.n_in() || ldr % 4 != 0 || lcq < w.Q || lcq % 64 != 0) return hipErrorInvalidValue;
    const dim3 grid((unsigned)M);
    if (prec)
        hipLaunchKernelGGL((latent_prepare_kernel<1>), grid, dim3(256), 0, s, w, qnorm, kvnorm, freq, raw, ldr, cache, pos0, cq, lcq);
    else
        hipLaunchKernelGGL((latent_prepare_kernel<0>), grid, dim3(256), 0, s, w, qnorm, kvnorm, freq, raw, ldr, cache, pos0, cq, lcq);
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------------------
// queries through k_up^T: workgroup (head, 128 columns of the latent, token); 16 threads share 8 columns, each every 16th
// element of the head.  One more column block makes the head's rotated part, and there, in a decode step, one more "head" the
// token's own cache row.
// ---------------------------------------------------------------------------------------------------------------
#define LQ_COLS 128
#define LQ_U 8  // rows a thread fetches together
__global__ __launch_bounds__(256) void latent_query_kernel(LatentShape w, const float *freq, const float *q, const uint16_t *ukv, int ldu,
                                                           float *qa, int pos0, const DecodeCtl *ctl, const float *in, const float *kvnorm,
                                                           float *cache) {
    extern __shared__ __align__(16) float s_mem[];
    __shared__ float s_acc[16][LQ_COLS + 4];
    const int h = blockIdx.x, m = blockIdx.z, t = threadIdx.x, c0 = blockIdx.y * LQ_COLS;
    if (blockIdx.y == gridDim.y - 1) {
        const int pos = ctl ? ctl->pos : pos0 + m;
        if (h == w.H) {
            lat_cache_row(w, kvnorm, freq, in + w.off_kv(), pos, cache + (int64_t)pos * w.ld(), s_acc[0]);
        } else if (t < 64) {
            float *dst = qa + ((int64_t)m * w.H + h) * w.ld() + w.Cp();
            l_rotate_norm(q + ((int64_t)m * w.H + h) * w.hq() + w.D, dst, w.R, w.rot, w.rot_half, freq, pos, 0, 0.0f, t);
            for (int i = w.R + t; i < w.Rp(); i += 64) dst[i] = 0.0f;
        }
        return;
    }
    if (h == w.H) return;
    const float *src = q + ((int64_t)m * w.H + h) * w.hq();
    float *dst = qa + ((int64_t)m * w.H + h) * w.ld();
    // the matrix's rows are under way before anything is waited for (ldu a multiple of 64, zero from C on)
    const int cg = t & 15, dg = t >> 4, c = c0 + 8 * cg;
    const uint16_t *rows = ukv + (int64_t)h * w.D * ldu + c;
    uint4 u[LQ_U];
    auto fetch = [&](int d0) {
#pragma unroll
        for (int k = 0; k < LQ_U; k++) {
            const int d = d0 + dg + 16 * k;
            u[k] = c < ldu && d < w.D ? *(const uint4 *)(rows + (int64_t)d * ldu) : make_uint4(0, 0, 0, 0);
        }
    };
    fetch(0);
    for (int i = t; i < w.D; i += 256) s_mem[i] = src[i];
    __syncthreads();
    float acc[8];
#pragma unroll
    for (int e = 0; e < 8; e++) acc[e] = 0.0f;
    for (int d0 = 0; d0 < w.D; d0 += 16 * LQ_U) {
        if (d0) fetch(d0);
#pragma unroll
        for (int k = 0; k < LQ_U; k++) {
            const int d = d0 + dg + 16 * k;
            const uint4 v = u[k];
            const float x = d < w.D ? s_mem[d] : 0.0f;
            acc[0] = fmaf(l_bf16_lo(v.x), x, acc[0]);
            acc[1] = fmaf(l_bf16_hi(v.x), x, acc[1]);
            acc[2] = fmaf(l_bf16_lo(v.y), x, acc[2]);
            acc[3] = fmaf(l_bf16_hi(v.y), x, acc[3]);
            acc[4] = fmaf(l_bf16_lo(v.z), x, acc[4]);
            acc[5] = fmaf(l_bf16_hi(v.z), x, acc[5]);
            acc[6] = fmaf(l_bf16_lo(v.w), x, acc[6]);
            acc[7] = fmaf(l_bf16_hi(v.w), x, acc[7]);
        }
    }
#pragma unroll
    for (int e = 0; e < 8; e++) s_acc[dg][8 * cg + e] = acc[e];
    __syncthreads();
    if (t < LQ_COLS && c0 + t < w.Cp()) {
        float v = 0.0f;
#pragma unroll
        for (int g = 0; g < 16; g++) v += s_acc[g][t];
        dst[c0 + t] = v;
    }
}
hipError_t k_latent_query(hipStream_t s, const LatentShape &w, const float *freq, const float *q, const uint16_t *ukv, int ldu,
                          float *qa, int M, int pos0, const DecodeCtl *ctl, const float *in, const float *kvnorm, float *cache) {
    if (M < 1 || ldu % 64 != 0 || ldu < w.C || (ctl && (M != 1 || !in || !cache))) return hipErrorInvalidValue;
    const dim3 grid((unsigned)(w.H + (ctl ? 1 : 0)), (unsigned)((w.Cp() + LQ_COLS - 1) / LQ_COLS + 1), (unsigned)M);
    hipLaunchKernelGGL(latent_query_kernel, grid, dim3(256), w.D * sizeof(float), s, w, freq, q, ukv, ldu, qa, pos0, ctl, in, kvnorm, cache);
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------------------
// Scores and value sums on the cached rows: workgroup (run of keys, 16 columns), a column being a (token, head).  Keys go 32 at
// a time.  The scores' contraction (the row's elements, 16 at a time) is shared out among the eight wavefronts and their parts
// are added in LDS; every wavefront then has the 32 x 16 scores in registers, in the layout that is the second product's
// operand when its contraction takes key 4 (lane / 16) + r in step r, and sums its own 64-element blocks of the latent:
// wavefront v the blocks v, v + 8, ...
//   v_mfma_f32_16x16x4_f32: operands hold (row or column lane % 16, k = lane / 16), the result (row 4 (lane / 16) + r, column
//   lane % 16); an operand's four consecutive elements of one 16-byte load serve four products.
// ---------------------------------------------------------------------------------------------------------------
#define LA_WAVES 8
#define LA_J 5  // 16-element steps of the scores' contraction a wavefront fetches together: rows of up to 640 elements
template <int NB>
__global__ __launch_bounds__(64 * LA_WAVES) void latent_attend_kernel(LatentShape w, const float *qa, const float *cache, float *part, int n_cols,
                                                            int pos0, const DecodeCtl *ctl, int n_split) {
    extern __shared__ __align__(16) float s_q[];  // [16][ld + 4]
    __shared__ float s_sc[2][LA_WAVES][8][64];
    const int t = threadIdx.x, lane = t & 63, wave = __builtin_amdgcn_readfirstlane(t >> 6), g = lane >> 4, col = lane & 15;
    const int ld = w.ld(), Cp = w.Cp(), qs = ld + 4, st = Cp + 4;
    const int c0 = 16 * blockIdx.y;
    // the columns' queries, 32 threads a column (columns past the last one repeat it; not stored)
    constexpr int QT = 4 * LA_WAVES, QE = 4 * QT;
    const int qc = t / QT, qe = 4 * (t % QT);
    const float *qsrc = qa + (int64_t)min(c0 + qc, n_cols - 1) * ld;
    float4 qr[LA_J];
#pragma unroll
    for (int u = 0; u < LA_J; u++) qr[u] = *(const float4 *)(qsrc + min(qe + QE * u, ld - 4));
    const int first = ctl ? ctl->pos : pos0;
    const int n_keys = first + min(c0 + 15, n_cols - 1) / w.H + 1;
    const int run = ((n_keys + n_split - 1) / n_split + 31) / 32 * 32, k0 = run * (int)blockIdx.x, k1 = min(k0 + run, n_keys);
    if (k0 >= k1) {
        if (t < 16 && c0 + t < n_cols) {
            float *p = part + ((int64_t)(c0 + t) * n_split + blockIdx.x) * st;
            p[0] = -INFINITY;
            p[1] = 0.0f;
        }
        return;
    }
    // the latents of the second product: keys kb + 4 g + r and 16 further, elements 64 (wave + 8 b) + 4 col ..; of the first:
    // keys kb + col and 16 further, elements 16 j + 4 g .., j = wave, wave + 8, ...
    float4 ka[LA_J], kc[LA_J], va[NB][8];
    auto key = [&](int k) { return cache + (int64_t)min(k, k1 - 1) * ld; };
    auto fetch_k = [&](int kb) {
        const float *a = key(kb + col) + 4 * g, *c = key(kb + 16 + col) + 4 * g;
#pragma unroll
        for (int u = 0; u < LA_J; u++) {
            const int at = min(16 * (wave + LA_WAVES * u), ld - 16);  // (a step past the row is not used)
            ka[u] = *(const float4 *)(a + at);
            kc[u] = *(const float4 *)(c + at);
        }
    };
    auto fetch_v = [&](int kb) {
#pragma unroll
        for (int r = 0; r < 8; r++) {
            const float *row = key(kb + 16 * (r >> 2) + 4 * g + (r & 3));
#pragma unroll
            for (int b = 0; b < NB; b++) {
                va[b][r] = *(const float4 *)(row + min(64 * (wave + LA_WAVES * b) + 4 * col, Cp - 4));  // (beyond Cp: not stored)
            }
        }
    };
    fetch_k(k0);
    fetch_v(k0);
    const int mine = c0 + col, limit = mine < n_cols ? min(first + mine / w.H, k1 - 1) : -1;  // last key this lane's column sees
#pragma unroll
    for (int u = 0; u < LA_J; u++)
        if (qe + QE * u < ld) *(float4 *)(s_q + qc * qs + qe + QE * u) = qr[u];
    for (int e = qe + QE * LA_J; e < ld; e += QE) *(float4 *)(s_q + qc * qs + e) = *(const float4 *)(qsrc + e);
    __syncthreads();
    lat_f32x4 o[NB][4];
#pragma unroll
    for (int b = 0; b < NB; b++)
#pragma unroll
        for (int i = 0; i < 4; i++) o[b][i] = lat_f32x4{0.f, 0.f, 0.f, 0.f};
    float mrun = -INFINITY, lrun = 0.0f;
    int stage = 0;
    for (int kb = k0; kb < k1; kb += 32, stage ^= 1) {
        lat_f32x4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = {0.f, 0.f, 0.f, 0.f};
        const float *qp = s_q + col * qs + 4 * g;
        auto score = [&](float4 x, float4 y, int j) {
            const float4 q = *(const float4 *)(qp + 16 * j);
            s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, q.x, s0, 0, 0, 0);
            s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(y.x, q.x, s1, 0, 0, 0);
            s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, q.y, s0, 0, 0, 0);
            s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(y.y, q.y, s1, 0, 0, 0);
            s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, q.z, s0, 0, 0, 0);
            s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(y.z, q.z, s1, 0, 0, 0);
            s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, q.w, s0, 0, 0, 0);
            s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(y.w, q.w, s1, 0, 0, 0);
        };
#pragma unroll
        for (int u = 0; u < LA_J; u++)
            if (16 * (wave + LA_WAVES * u) < ld) score(ka[u], kc[u], wave + LA_WAVES * u);
        for (int j = wave + LA_WAVES * LA_J; 16 * j < ld; j += LA_WAVES)
            score(*(const float4 *)(key(kb + col) + 4 * g + 16 * j), *(const float4 *)(key(kb + 16 + col) + 4 * g + 16 * j), j);
        if (kb + 32 < k1) fetch_k(kb + 32);
#pragma unroll
        for (int r = 0; r < 4; r++) {
            s_sc[stage][wave][r][lane] = s0[r];
            s_sc[stage][wave][4 + r][lane] = s1[r];
        }
        __syncthreads();  // (the other stage is written again only behind the next one)
        float p[8], mx = -INFINITY;
#pragma unroll
        for (int r = 0; r < 8; r++) {
            float v = 0.0f;
#pragma unroll
            for (int i = 0; i < LA_WAVES; i++) v += s_sc[stage][i][r][lane];
            p[r] = kb + 16 * (r >> 2) + 4 * g + (r & 3) <= limit ? v * w.scale : -INFINITY;
            mx = fmaxf(mx, p[r]);
        }
        mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
        mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
        const float mnew = fmaxf(mrun, mx), alpha = mnew == -INFINITY ? 1.0f : expf(mrun - mnew);
        float sum = 0.0f;
#pragma unroll
        for (int r = 0; r < 8; r++) {
            p[r] = p[r] == -INFINITY ? 0.0f : expf(p[r] - mnew);
            sum += p[r];
        }
        sum += __shfl_xor(sum, 16, WAVE);
        sum += __shfl_xor(sum, 32, WAVE);
        lrun = lrun * alpha + sum;
        mrun = mnew;
#pragma unroll
        for (int b = 0; b < NB; b++) {
#pragma unroll
            for (int i = 0; i < 4; i++) o[b][i] *= alpha;
#pragma unroll
            for (int r = 0; r < 8; r++) {
                o[b][0] = __builtin_amdgcn_mfma_f32_16x16x4f32(va[b][r].x, p[r], o[b][0], 0, 0, 0);
                o[b][1] = __builtin_amdgcn_mfma_f32_16x16x4f32(va[b][r].y, p[r], o[b][1], 0, 0, 0);
                o[b][2] = __builtin_amdgcn_mfma_f32_16x16x4f32(va[b][r].z, p[r], o[b][2], 0, 0, 0);
                o[b][3] = __builtin_amdgcn_mfma_f32_16x16x4f32(va[b][r].w, p[r], o[b][3], 0, 0, 0);
            }
        }
        if (kb + 32 < k1) fetch_v(kb + 32);
    }
    if (mine >= n_cols) return;
    float *dst = part + ((int64_t)mine * n_split + blockIdx.x) * st;
    if (wave == 0 && g == 0) {
        dst[0] = mrun;
        dst[1] = lrun;
    }
#pragma unroll
    for (int b = 0; b < NB; b++)
#pragma unroll
        for (int r = 0; r < 4; r++) {  // row 4 g + r of result i is element 4 (4 g + r) + i of the block
            const int c = 64 * (wave + LA_WAVES * b) + 4 * (4 * g + r);
            if (c < Cp) *(float4 *)(dst + 4 + c) = make_float4(o[b][0][r], o[b][1][r], o[b][2][r], o[b][3][r]);
        }
}
hipError_t k_latent_attend(hipStream_t s, const LatentShape &w, const float *qa, const float *cache, float *part, int M, int pos0,
                           const DecodeCtl *ctl) {
    if (M < 1 || w.C > L_LATENT_MAX_RANK || (!ctl && (pos0 < 0 || pos0 + M > w.seq_len)) || (ctl && M != 1)) return hipErrorInvalidValue;
    const int cols = M * w.H, ns = latent_splits(cols);
    const size_t lds = (size_t)16 * (w.ld() + 4) * sizeof(float);
    if (lds > 100 * 1024) return hipErrorInvalidValue;
    const int nb = ((w.Cp() + 63) / 64 + LA_WAVES - 1) / LA_WAVES;  // at most 2
    const dim3 grid((unsigned)ns, (unsigned)((cols + 15) / 16));
#define GO(N)                                                                                                                          \
    do {                                                                                                                               \
        if (lds > 32 * 1024) {                                                                                                         \
            const hipError_t e = hipFuncSetAttribute((const void *)latent_attend_kernel<N>, hipFuncAttributeMaxDynamicSharedMemorySize, \
                                                     100 * 1024);                                                                      \
            if (e != hipSuccess) return e;                                                                                             \
        }                                                                                                                              \
        hipLaunchKernelGGL((latent_attend_kernel<N>), grid, dim3(64 * LA_WAVES), lds, s, w, qa, cache, part, cols, pos0, ctl, ns);               \
    } while (0)
    if (nb == 1)
        GO(1);
    else
        GO(2);
#undef GO
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------------------
// joins the runs' sums and applies v_up and the gate: workgroup (head, 32 of its value elements, token)
// ---------------------------------------------------------------------------------------------------------------
#define LV_ROWS 32
#define LV_THREADS 1024
#define LV_U 12  // runs a thread fetches together
template <int PREC>
__global__ __launch_bounds__(LV_THREADS) void latent_value_kernel(LatentShape w, const float *part, const uint16_t *ukv, int ldu,
                                                                  const float *raw, int64_t ldr, void *outa, int64_t lda, int64_t cols,
                                                                  int n_split) {
    extern __shared__ __align__(16) float s_mem[];
    __shared__ float s_f[L_LATENT_SPLITS];
    __shared__ int s_used;
    const int h = blockIdx.x, e0 = blockIdx.y * LV_ROWS, m = blockIdx.z, t = threadIdx.x, lane = t & 63, wave = t >> 6;
    const int Cp = w.Cp(), st = Cp + 4, nq = Cp / 4, ng = LV_THREADS / nq;  // (Cp <= 1024)
    float *s_c = s_mem, *s_acc = s_c + ldu;
    const float *p = part + ((int64_t)m * w.H + h) * n_split * st;
    // this wavefront's rows and this thread's part of the sums are under way before anything is waited for
    constexpr int RW = LV_ROWS / (LV_THREADS / 64);
    const uint16_t *rows = ukv + ((int64_t)w.H * w.D + (int64_t)h * w.V) * ldu;
    uint4 wr[RW];
#pragma unroll
    for (int i = 0; i < RW; i++) {
        const int e = e0 + wave * RW + i;
        wr[i] = e < w.V && 8 * lane < ldu ? *(const uint4 *)(rows + (int64_t)e * ldu + 8 * lane) : make_uint4(0, 0, 0, 0);
    }
    const int cq = t % nq, cg = t / nq;
    float4 v[LV_U];
    auto fetch = [&](int i0) {
#pragma unroll
        for (int u = 0; u < LV_U; u++) {
            const int i = i0 + cg + u * ng;
            v[u] = cg < ng && i < n_split ? *(const float4 *)(p + (int64_t)i * st + 4 + 4 * cq) : lat_zero4();
        }
    };
    fetch(0);
    if (t < 64) {
        constexpr int N = L_LATENT_SPLITS / 64;
        float mv[N], lv[N], mx = -INFINITY, l = 0.0f;
#pragma unroll
        for (int u = 0; u < N; u++) {
            const int i = t + 64 * u;
            mv[u] = i < n_split ? p[(int64_t)i * st] : -INFINITY;
            lv[u] = i < n_split ? p[(int64_t)i * st + 1] : 0.0f;
            mx = fmaxf(mx, mv[u]);
        }
        mx = wave_max_f32(mx);
#pragma unroll
        for (int u = 0; u < N; u++) {
            mv[u] = mv[u] == -INFINITY ? 0.0f : expf(mv[u] - mx);
            l = fmaf(mv[u], lv[u], l);
        }
        l = l_wave_sum(l);
#pragma unroll
        for (int u = 0; u < N; u++) s_f[t + 64 * u] = mv[u] / l;
        int used = 0;  // runs up to the last one with keys
#pragma unroll
        for (int u = 0; u < N; u++) {
            const unsigned long long b = __ballot(mv[u] != 0.0f);
            if (b) used = 64 * u + 64 - __builtin_clzll(b);
        }
        if (t == 0) s_used = used;
    }
    for (int i = Cp + t; i < ldu; i += LV_THREADS) s_c[i] = 0.0f;
    __syncthreads();
    if (cg < ng) {
        float4 a = lat_zero4();
        for (int i0 = 0; i0 < s_used; i0 += LV_U * ng) {
            if (i0) fetch(i0);
#pragma unroll
            for (int u = 0; u < LV_U; u++) {
                const int i = i0 + cg + u * ng;
                const float f = i < n_split ? s_f[i] : 0.0f;
                if (f == 0.0f) continue;  // (a run without keys, whose sums were not written)
                a.x = fmaf(f, v[u].x, a.x);
                a.y = fmaf(f, v[u].y, a.y);
                a.z = fmaf(f, v[u].z, a.z);
                a.w = fmaf(f, v[u].w, a.w);
            }
        }
        *(float4 *)(s_acc + cg * Cp + 4 * cq) = a;
    }
    __syncthreads();
    for (int c = t; c < Cp; c += LV_THREADS) {
        float a = 0.0f;
        for (int i = 0; i < ng; i++) a += s_acc[i * Cp + c];
        s_c[c] = a;
    }
    __syncthreads();
    float acc[RW];
#pragma unroll
    for (int i = 0; i < RW; i++) acc[i] = 0.0f;
    for (int k = 8 * lane; k < ldu; k += 512) {
        const float4 xa = *(const float4 *)(s_c + k), xb = *(const float4 *)(s_c + k + 4);
#pragma unroll
        for (int i = 0; i < RW; i++) {
            const int e = e0 + wave * RW + i;
            uint4 x = wr[i];
            if (k >= 512) x = e < w.V ? *(const uint4 *)(rows + (int64_t)e * ldu + k) : make_uint4(0, 0, 0, 0);
            acc[i] = fmaf(l_bf16_lo(x.x), xa.x, acc[i]);
            acc[i] = fmaf(l_bf16_hi(x.x), xa.y, acc[i]);
            acc[i] = fmaf(l_bf16_lo(x.y), xa.z, acc[i]);
            acc[i] = fmaf(l_bf16_hi(x.y), xa.w, acc[i]);
            acc[i] = fmaf(l_bf16_lo(x.z), xb.x, acc[i]);
            acc[i] = fmaf(l_bf16_hi(x.z), xb.y, acc[i]);
            acc[i] = fmaf(l_bf16_lo(x.w), xb.z, acc[i]);
            acc[i] = fmaf(l_bf16_hi(x.w), xb.w, acc[i]);
        }
    }
#pragma unroll
    for (int i = 0; i < RW; i++) {
        const float a = l_wave_sum(acc[i]);
        const int e = e0 + wave * RW + i;
        if (lane == i && e < w.V) {
            const int64_t at = (int64_t)h * w.V + e;
            l_store_act<PREC>(outa, m * lda + at, w.gated ? a * l_sigmoid(raw[(int64_t)m * ldr + w.off_g() + at]) : a);
        }
    }
    if (h == w.H - 1 && blockIdx.y == 0)
        for (int64_t i = (int64_t)w.H * w.V + t; i < cols; i += LV_THREADS) l_store_act<PREC>(outa, m * lda + i, 0.0f);
}
hipError_t k_latent_value(hipStream_t s, const LatentShape &w, const float *part, const uint16_t *ukv, int ldu, const float *raw,
                          int64_t ldr, int M, void *outa, int64_t lda, int64_t cols, int prec) {
    if (M < 1 || w.C > L_LATENT_MAX_RANK || ldu % 64 != 0 || ldu < w.C || cols > lda || cols < (int64_t)w.H * w.V) return hipErrorInvalidValue;
    const int ns = latent_splits((int64_t)M * w.H), nq = w.Cp() / 4, ng = LV_THREADS / nq;
    const size_t lds = ((size_t)ldu + (size_t)ng * w.Cp()) * sizeof(float);
    const dim3 grid((unsigned)w.H, (unsigned)((w.V + LV_ROWS - 1) / LV_ROWS), (unsigned)M);
    if (prec)
        hipLaunchKernelGGL((latent_value_kernel<1>), grid, dim3(LV_THREADS), lds, s, w, part, ukv, ldu, raw, ldr, outa, lda, cols, ns);
    else
        hipLaunchKernelGGL((latent_value_kernel<0>), grid, dim3(LV_THREADS), lds, s, w, part, ukv, ldu, raw, ldr, outa, lda, cols, ns);
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------------------
// operands of the matrix-core attention
// ---------------------------------------------------------------------------------------------------------------
// one wavefront per (token, head)
__global__ __launch_bounds__(256) void latent_heads_kernel(LatentShape w, const float *freq, const float *q, uint16_t *qb, int hs, int M,
                                                           int pos0) {
    extern __shared__ __align__(16) float s_mem[];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, m = blockIdx.y, h = blockIdx.x * 4 + wave;
    if (h >= w.H) return;
    const int64_t u = (int64_t)m * w.H + h;
    const float *src = q + u * w.hq();
    float *x = s_mem + wave * (w.R + 1);
    l_rotate_norm(src + w.D, x, w.R, w.rot, w.rot_half, freq, pos0 + m, 0, 0.0f, lane);
    __builtin_amdgcn_wave_barrier();
    for (int i = 2 * lane; i < hs; i += 128) {
        float v[2];
#pragma unroll
        for (int e = 0; e < 2; e++) v[e] = i + e < w.D ? src[i + e] : i + e < w.hq() ? x[i + e - w.D] : 0.0f;
        *(uint32_t *)(qb + u * hs + i) = l_pack_bf16(v[0], v[1]);
    }
}
hipError_t k_latent_heads(hipStream_t s, const LatentShape &w, const float *freq, const float *q, uint16_t *qb, int hs, int M, int pos0) {
    if (M < 1 || hs < w.hq() || hs % 2 != 0) return hipErrorInvalidValue;
    hipLaunchKernelGGL(latent_heads_kernel, dim3((unsigned)((w.H + 3) / 4), (unsigned)M), dim3(256), 4 * (w.R + 1) * sizeof(float), s, w, freq,
                       q, qb, hs, M, pos0);
    return hipGetLastError();
}

// one thread per pair of elements
__global__ __launch_bounds__(256) void latent_rows_kernel(LatentShape w, const float *cache, int pos0, int n, uint16_t *outa, int64_t lda) {
    const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x, half = lda / 2, r = idx / half;
    const int i = 2 * (int)(idx - r * half);
    if (r >= n) return;
    const float *row = cache + (pos0 + r) * w.ld();
    *(uint32_t *)(outa + r * lda + i) = l_pack_bf16(i < w.C ? row[i] : 0.0f, i + 1 < w.C ? row[i + 1] : 0.0f);
}
hipError_t k_latent_rows(hipStream_t s, const LatentShape &w, const float *cache, int pos0, int n, uint16_t *outa, int64_t lda) {
    if (n < 1 || pos0 < 0 || pos0 + n > w.seq_len || lda % 2 != 0 || lda < w.C) return hipErrorInvalidValue;
    const int64_t total = (int64_t)n * lda / 2;
    hipLaunchKernelGGL(latent_rows_kernel, dim3((unsigned)((total + 255) / 256)), dim3(256), 0, s, w, cache, pos0, n, outa, lda);
    return hipGetLastError();
}
