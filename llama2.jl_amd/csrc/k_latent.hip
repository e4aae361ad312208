// Attention over a cached latent: the cache holds one normed latent and one rotated key part per position, which all heads
// share.  For few tokens the queries are taken through k_up^T, so that scores and value sums are formed on the cached rows
// themselves (fp32 matrix cores), and v_up is applied once per token.  Everything is fp32; matrices are bf16 rows.
#include "layered_dev.h"

typedef float lat_f32x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float4 lat_zero4() { return make_float4(0.f, 0.f, 0.f, 0.f); }

// ---------------------------------------------------------------------------------------------------------------
// a position's cache row, by one wavefront: src holds the projected [C | R] elements
// ---------------------------------------------------------------------------------------------------------------
__device__ __forceinline__ void lat_cache_row(const LatentShape &w, const float *kvnorm, const float *freq, const float *src, int pos,
                                              float *row, int lane) {
    float ss = 0.0f;
    for (int i = lane; i < w.C; i += 64) ss = fmaf(src[i], src[i], ss);
    const float r = 1.0f / sqrtf(l_wave_sum(ss) / (float)w.C + w.eps);
    for (int i = lane; i < w.Cp(); i += 64) row[i] = i < w.C ? src[i] * r * kvnorm[i] : 0.0f;
    l_rotate_norm(src + w.C, row + w.Cp(), w.R, w.rot, w.rot_half, freq, pos, 0, 0.0f, lane);
    for (int i = w.R + lane; i < w.Rp(); i += 64) row[w.Cp() + i] = 0.0f;
}

// many tokens: one wavefront each
template <int PREC>
__global__ __launch_bounds__(256) void latent_prepare_kernel(LatentShape w, const float *qnorm, const float *kvnorm, const float *freq,
                                                             const float *raw, int64_t ldr, float *cache, int M, int pos0, void *cq,
                                                             int64_t lcq) {
    const int lane = threadIdx.x & 63, m = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (m >= M) return;
    const float *src = raw + (int64_t)m * ldr;
    float ss = 0.0f;
    for (int i = lane; i < w.Q; i += 64) ss = fmaf(src[i], src[i], ss);
    const float r = 1.0f / sqrtf(l_wave_sum(ss) / (float)w.Q + w.eps);
    for (int64_t i = lane; i < lcq; i += 64) l_store_act<PREC>(cq, m * lcq + i, i < w.Q ? src[i] * r * qnorm[i] : 0.0f);
    lat_cache_row(w, kvnorm, freq, src + w.off_kv(), pos0 + m, cache + (int64_t)(pos0 + m) * w.ld(), lane);
}
hipError_t k_latent_prepare(hipStream_t s, const LatentShape &w, const float *qnorm, const float *kvnorm, const float *freq,
                            const float *raw, int64_t ldr, float *cache, int M, int pos0, void *cq, int64_t lcq, int prec) {
    if (M < 1 || pos0 < 0 || pos0 + M > w.seq_len || ldr < w.n_in() || lcq < w.Q) return hipErrorInvalidValue;
    const dim3 grid((unsigned)((M + 3) / 4));
    if (prec)
        hipLaunchKernelGGL((latent_prepare_kernel<1>), grid, dim3(256), 0, s, w, qnorm, kvnorm, freq, raw, ldr, cache, M, pos0, cq, lcq);
    else
        hipLaunchKernelGGL((latent_prepare_kernel<0>), grid, dim3(256), 0, s, w, qnorm, kvnorm, freq, raw, ldr, cache, M, pos0, cq, lcq);
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------------------
// queries through k_up^T: workgroup (head, 128 columns of the latent, token); 16 threads share 8 columns, each every 16th
// element of the head.  The column block 0 also makes the head's rotated part, and in a decode step one more "head" the
// token's own cache row.
// ---------------------------------------------------------------------------------------------------------------
#define LQ_COLS 128
__global__ __launch_bounds__(256) void latent_query_kernel(LatentShape w, const float *freq, const float *q, const uint16_t *ukv, int ldu,
                                                           float *qa, int pos0, const DecodeCtl *ctl, const float *in, const float *kvnorm,
                                                           float *cache) {
    extern __shared__ __align__(16) float s_mem[];
    __shared__ float s_acc[16][LQ_COLS + 4];
    const int h = blockIdx.x, m = blockIdx.z, t = threadIdx.x, c0 = blockIdx.y * LQ_COLS;
    const int pos = ctl ? ctl->pos : pos0 + m;
    if (h == w.H) {
        if (blockIdx.y == 0 && t < 64) lat_cache_row(w, kvnorm, freq, in + w.off_kv(), pos, cache + (int64_t)pos * w.ld(), t);
        return;
    }
    const float *src = q + ((int64_t)m * w.H + h) * w.hq();
    float *dst = qa + ((int64_t)m * w.H + h) * w.ld();
    if (blockIdx.y == 0 && t >= 192) {
        const int lane = t - 192;
        l_rotate_norm(src + w.D, dst + w.Cp(), w.R, w.rot, w.rot_half, freq, pos, 0, 0.0f, lane);
        for (int i = w.R + lane; i < w.Rp(); i += 64) dst[w.Cp() + i] = 0.0f;
    }
    const int cg = t & 15, dg = t >> 4, c = c0 + 8 * cg;
    for (int i = t; i < w.D; i += 256) s_mem[i] = src[i];
    __syncthreads();
    float acc[8];
#pragma unroll
    for (int e = 0; e < 8; e++) acc[e] = 0.0f;
    if (c < ldu) {  // (ldu a multiple of 64, zero from C on)
        const uint16_t *u = ukv + (int64_t)h * w.D * ldu + c;
#pragma unroll 8
        for (int d = dg; d < w.D; d += 16) {
            const uint4 v = *(const uint4 *)(u + (int64_t)d * ldu);
            const float x = s_mem[d];
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
    const dim3 grid((unsigned)(w.H + (ctl ? 1 : 0)), (unsigned)((w.Cp() + LQ_COLS - 1) / LQ_COLS), (unsigned)M);
    hipLaunchKernelGGL(latent_query_kernel, grid, dim3(256), w.D * sizeof(float), s, w, freq, q, ukv, ldu, qa, pos0, ctl, in, kvnorm, cache);
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------------------
// Scores and value sums on the cached rows: workgroup (run of keys, 16 columns), a column being a (token, head).  Keys go 32 at
// a time.  The scores' contraction (the row's elements, 16 at a time) is shared out among the four wavefronts and their parts
// are added in LDS; every wavefront then has the 32 x 16 scores in registers, in the layout that is the second product's
// operand when its contraction takes key 4 (lane / 16) + r in step r, and sums its own 64-element blocks of the latent:
// wavefront v the blocks v, v + 4, ...
//   v_mfma_f32_16x16x4_f32: operands hold (row or column lane % 16, k = lane / 16), the result (row 4 (lane / 16) + r, column
//   lane % 16); an operand's four consecutive elements of one 16-byte load serve four products.
// ---------------------------------------------------------------------------------------------------------------
template <int NB>
__global__ __launch_bounds__(256) void latent_attend_kernel(LatentShape w, const float *qa, const float *cache, float *part, int n_cols,
                                                            int pos0, const DecodeCtl *ctl, int n_split) {
    extern __shared__ __align__(16) float s_q[];  // [16][ld + 4]
    __shared__ float s_sc[2][4][8][64];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, g = lane >> 4, col = lane & 15;
    const int ld = w.ld(), Cp = w.Cp(), qs = ld + 4, st = Cp + 4;
    const int c0 = 16 * blockIdx.y, first = ctl ? ctl->pos : pos0;
    const int n_keys = first + min(c0 + 15, n_cols - 1) / w.H + 1;
    const int run = ((n_keys + n_split - 1) / n_split + 15) / 16 * 16, k0 = run * (int)blockIdx.x, k1 = min(k0 + run, n_keys);
    if (k0 >= k1) {
        if (t < 16 && c0 + t < n_cols) {
            float *p = part + ((int64_t)(c0 + t) * n_split + blockIdx.x) * st;
            p[0] = -INFINITY;
            p[1] = 0.0f;
        }
        return;
    }
    const int mine = c0 + col, limit = mine < n_cols ? min(first + mine / w.H, k1 - 1) : -1;  // last key this lane's column sees
    for (int i = 4 * t; i < 16 * ld; i += 1024) {
        const int c = i / ld, e = i - c * ld;
        *(float4 *)(s_q + c * qs + e) = c0 + c < n_cols ? *(const float4 *)(qa + (int64_t)(c0 + c) * ld + e) : lat_zero4();
    }
    __syncthreads();
    lat_f32x4 o[NB][4];
#pragma unroll
    for (int b = 0; b < NB; b++)
#pragma unroll
        for (int i = 0; i < 4; i++) o[b][i] = lat_f32x4{0.f, 0.f, 0.f, 0.f};
    float mrun = -INFINITY, lrun = 0.0f;
    int stage = 0;
    for (int kb = k0; kb < k1; kb += 32, stage ^= 1) {
        const float *ka = cache + (int64_t)min(kb + col, k1 - 1) * ld + 4 * g, *kc = cache + (int64_t)min(kb + 16 + col, k1 - 1) * ld + 4 * g;
        // the latents of the second product: keys kb + 4 g + r and 16 further, elements 64 (wave + 4 b) + 4 col ..
        float4 va[NB][8];
#pragma unroll
        for (int r = 0; r < 8; r++) {
            const float *row = cache + (int64_t)min(kb + 16 * (r >> 2) + 4 * g + (r & 3), k1 - 1) * ld;
#pragma unroll
            for (int b = 0; b < NB; b++) {
                const int c = 64 * (wave + 4 * b) + 4 * col;
                va[b][r] = c < Cp ? *(const float4 *)(row + c) : lat_zero4();
            }
        }
        lat_f32x4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = {0.f, 0.f, 0.f, 0.f};
        const float *qp = s_q + col * qs + 4 * g;
#pragma unroll 4
        for (int j = wave; 16 * j < ld; j += 4) {
            const float4 x = *(const float4 *)(ka + 16 * j), y = *(const float4 *)(kc + 16 * j), q = *(const float4 *)(qp + 16 * j);
            s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, q.x, s0, 0, 0, 0);
            s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(y.x, q.x, s1, 0, 0, 0);
            s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, q.y, s0, 0, 0, 0);
            s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(y.y, q.y, s1, 0, 0, 0);
            s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, q.z, s0, 0, 0, 0);
            s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(y.z, q.z, s1, 0, 0, 0);
            s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, q.w, s0, 0, 0, 0);
            s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(y.w, q.w, s1, 0, 0, 0);
        }
#pragma unroll
        for (int r = 0; r < 4; r++) {
            s_sc[stage][wave][r][lane] = s0[r];
            s_sc[stage][wave][4 + r][lane] = s1[r];
        }
        __syncthreads();  // (the other stage is written again only behind the next one)
        float p[8], mx = -INFINITY;
#pragma unroll
        for (int r = 0; r < 8; r++) {
            const float v = s_sc[stage][0][r][lane] + s_sc[stage][1][r][lane] + s_sc[stage][2][r][lane] + s_sc[stage][3][r][lane];
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
            const int c = 64 * (wave + 4 * b) + 4 * (4 * g + r);
            if (c < Cp) *(float4 *)(dst + 4 + c) = make_float4(o[b][0][r], o[b][1][r], o[b][2][r], o[b][3][r]);
        }
}
hipError_t k_latent_attend(hipStream_t s, const LatentShape &w, const float *qa, const float *cache, float *part, int M, int pos0,
                           const DecodeCtl *ctl) {
    if (M < 1 || w.C > L_LATENT_MAX_RANK || (!ctl && (pos0 < 0 || pos0 + M > w.seq_len)) || (ctl && M != 1)) return hipErrorInvalidValue;
    const int cols = M * w.H, ns = latent_splits(cols);
    const size_t lds = (size_t)16 * (w.ld() + 4) * sizeof(float);
    if (lds > 100 * 1024) return hipErrorInvalidValue;
    const int nb = ((w.Cp() + 63) / 64 + 3) / 4;
    const dim3 grid((unsigned)ns, (unsigned)((cols + 15) / 16));
#define GO(N)                                                                                                                          \
    do {                                                                                                                               \
        if (lds > 32 * 1024) {                                                                                                         \
            const hipError_t e = hipFuncSetAttribute((const void *)latent_attend_kernel<N>, hipFuncAttributeMaxDynamicSharedMemorySize, \
                                                     100 * 1024);                                                                      \
            if (e != hipSuccess) return e;                                                                                             \
        }                                                                                                                              \
        hipLaunchKernelGGL((latent_attend_kernel<N>), grid, dim3(256), lds, s, w, qa, cache, part, cols, pos0, ctl, ns);               \
    } while (0)
    if (nb == 1)
        GO(1);
    else if (nb == 2)
        GO(2);
    else
        GO(4);
#undef GO
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------------------
// joins the runs' sums and applies v_up and the gate: workgroup (head, 32 of its value elements, token)
// ---------------------------------------------------------------------------------------------------------------
#define LV_ROWS 32
template <int PREC>
__global__ __launch_bounds__(256) void latent_value_kernel(LatentShape w, const float *part, const uint16_t *ukv, int ldu, const float *raw,
                                                           int64_t ldr, void *outa, int64_t lda, int64_t cols, int n_split) {
    extern __shared__ __align__(16) float s_mem[];
    __shared__ float s_f[64];
    const int h = blockIdx.x, e0 = blockIdx.y * LV_ROWS, m = blockIdx.z, t = threadIdx.x, lane = t & 63, wave = t >> 6;
    const int Cp = w.Cp(), st = Cp + 4, nq = Cp / 4, ng = nq <= 256 ? 256 / nq : 1;  // (Cp <= 1024)
    float *s_c = s_mem, *s_acc = s_c + ldu;
    const float *p = part + ((int64_t)m * w.H + h) * n_split * st;
    // this wavefront's rows: their first chunks are under way while the sums are joined
    constexpr int RW = LV_ROWS / 4;
    const uint16_t *rows = ukv + ((int64_t)w.H * w.D + (int64_t)h * w.V) * ldu;
    uint4 wr[RW];
#pragma unroll
    for (int i = 0; i < RW; i++) {
        const int e = e0 + wave * RW + i;
        wr[i] = e < w.V && 8 * lane < ldu ? *(const uint4 *)(rows + (int64_t)e * ldu + 8 * lane) : make_uint4(0, 0, 0, 0);
    }
    if (t < 64) {  // (n_split <= 64)
        const float mv = t < n_split ? p[(int64_t)t * st] : -INFINITY;
        const float mx = wave_max_f32(mv), f = mv == -INFINITY ? 0.0f : expf(mv - mx);
        const float l = l_wave_sum(f != 0.0f ? f * p[(int64_t)t * st + 1] : 0.0f);
        s_f[t] = f / l;
    }
    for (int i = Cp + t; i < ldu; i += 256) s_c[i] = 0.0f;
    __syncthreads();
    const int cq = t % nq, cg = t / nq;
    if (cg < ng) {
        float4 a = lat_zero4();
#pragma unroll 8
        for (int i = cg; i < n_split; i += ng) {
            const float f = s_f[i];
            if (f == 0.0f) continue;  // (a run without keys, whose sums were not written)
            const float4 v = *(const float4 *)(p + (int64_t)i * st + 4 + 4 * cq);
            a.x = fmaf(f, v.x, a.x);
            a.y = fmaf(f, v.y, a.y);
            a.z = fmaf(f, v.z, a.z);
            a.w = fmaf(f, v.w, a.w);
        }
        *(float4 *)(s_acc + cg * Cp + 4 * cq) = a;
    }
    __syncthreads();
    for (int c = t; c < Cp; c += 256) {
        float v = 0.0f;
        for (int i = 0; i < ng; i++) v += s_acc[i * Cp + c];
        s_c[c] = v;
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
            uint4 v = wr[i];
            if (k >= 512) v = e < w.V ? *(const uint4 *)(rows + (int64_t)e * ldu + k) : make_uint4(0, 0, 0, 0);
            acc[i] = fmaf(l_bf16_lo(v.x), xa.x, acc[i]);
            acc[i] = fmaf(l_bf16_hi(v.x), xa.y, acc[i]);
            acc[i] = fmaf(l_bf16_lo(v.y), xa.z, acc[i]);
            acc[i] = fmaf(l_bf16_hi(v.y), xa.w, acc[i]);
            acc[i] = fmaf(l_bf16_lo(v.z), xb.x, acc[i]);
            acc[i] = fmaf(l_bf16_hi(v.z), xb.y, acc[i]);
            acc[i] = fmaf(l_bf16_lo(v.w), xb.z, acc[i]);
            acc[i] = fmaf(l_bf16_hi(v.w), xb.w, acc[i]);
        }
    }
#pragma unroll
    for (int i = 0; i < RW; i++) {
        const float v = l_wave_sum(acc[i]);
        const int e = e0 + wave * RW + i;
        if (lane == i && e < w.V) {
            const int64_t at = (int64_t)h * w.V + e;
            l_store_act<PREC>(outa, m * lda + at, w.gated ? v * l_sigmoid(raw[(int64_t)m * ldr + w.off_g() + at]) : v);
        }
    }
    if (h == w.H - 1 && blockIdx.y == 0)
        for (int64_t i = (int64_t)w.H * w.V + t; i < cols; i += 256) l_store_act<PREC>(outa, m * lda + i, 0.0f);
}
hipError_t k_latent_value(hipStream_t s, const LatentShape &w, const float *part, const uint16_t *ukv, int ldu, const float *raw,
                          int64_t ldr, int M, void *outa, int64_t lda, int64_t cols, int prec) {
    if (M < 1 || w.C > L_LATENT_MAX_RANK || ldu % 64 != 0 || ldu < w.C || cols > lda || cols < (int64_t)w.H * w.V) return hipErrorInvalidValue;
    const int ns = latent_splits((int64_t)M * w.H), nq = w.Cp() / 4, ng = nq <= 256 ? 256 / nq : 1;
    const size_t lds = ((size_t)ldu + (size_t)ng * w.Cp()) * sizeof(float);
    const dim3 grid((unsigned)w.H, (unsigned)((w.V + LV_ROWS - 1) / LV_ROWS), (unsigned)M);
    if (prec)
        hipLaunchKernelGGL((latent_value_kernel<1>), grid, dim3(256), lds, s, w, part, ukv, ldu, raw, ldr, outa, lda, cols, ns);
    else
        hipLaunchKernelGGL((latent_value_kernel<0>), grid, dim3(256), lds, s, w, part, ukv, ldu, raw, ldr, outa, lda, cols, ns);
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
