// One token through a bf16 matrix: a workgroup stages the input vector in LDS behind a fused prologue (norms, expert
// choice), its wavefronts stream whole matrix rows, two at a time, 16 bytes per lane and load, and a fused epilogue writes
// the results.  Activations and sums are fp32 throughout.
#include "layered_dev.h"

#define ROWS_THREADS 512
#define ROWS_WAVES 8
#define ROWS_MAX_EXPERTS 1024
#define ROWS_MAX_TOP 64

// element e of the staged vector: the two halves of every group of 8 lie in separate planes, so that the lanes of a
// wavefront, each reading 8 consecutive elements as two 16-byte words, touch consecutive words
__device__ __forceinline__ int xs_index(int e, int plane) { return ((e >> 2) & 1) * plane + ((e >> 3) << 2) + (e & 3); }

// one 16-byte chunk of each of a pair of rows against the staged vector
struct RowsChunk {
    uint4 p, q;
};
__device__ __forceinline__ void rows_load(RowsChunk &c, const uint16_t *w0, const uint16_t *w1, int k, int ld) {
    if (k < ld) {
        c.p = *(const uint4 *)(w0 + k);
        c.q = *(const uint4 *)(w1 + k);
    }
}
__device__ __forceinline__ void rows_fma(const RowsChunk &c, const float *xv, int plane, int k, int ld, float &acc0, float &acc1) {
    if (k >= ld) return;
    const uint4 p = c.p, q = c.q;
    const float4 xa = *(const float4 *)(xv + (k >> 1)), xb = *(const float4 *)(xv + plane + (k >> 1));
    acc0 = fmaf(l_bf16_lo(p.x), xa.x, acc0);
    acc1 = fmaf(l_bf16_lo(q.x), xa.x, acc1);
    acc0 = fmaf(l_bf16_hi(p.x), xa.y, acc0);
    acc1 = fmaf(l_bf16_hi(q.x), xa.y, acc1);
    acc0 = fmaf(l_bf16_lo(p.y), xa.z, acc0);
    acc1 = fmaf(l_bf16_lo(q.y), xa.z, acc1);
    acc0 = fmaf(l_bf16_hi(p.y), xa.w, acc0);
    acc1 = fmaf(l_bf16_hi(q.y), xa.w, acc1);
    acc0 = fmaf(l_bf16_lo(p.z), xb.x, acc0);
    acc1 = fmaf(l_bf16_lo(q.z), xb.x, acc1);
    acc0 = fmaf(l_bf16_hi(p.z), xb.y, acc0);
    acc1 = fmaf(l_bf16_hi(q.z), xb.y, acc1);
    acc0 = fmaf(l_bf16_lo(p.w), xb.z, acc0);
    acc1 = fmaf(l_bf16_lo(q.w), xb.z, acc1);
    acc0 = fmaf(l_bf16_hi(p.w), xb.w, acc0);
    acc1 = fmaf(l_bf16_hi(q.w), xb.w, acc1);
}

#define ROWS_V 4  // steps of 4 elements a thread of the staged vectors
#define ROWS_U 4  // chunks of a row pair fetched together: 2 rows x 4 KB per wavefront

// KSPLIT: the wavefronts share every pair of rows, each its part of the inputs (matrices with few rows)
template <int PRO, int EPI, bool KSPLIT>
__global__ __launch_bounds__(ROWS_THREADS) void rows_kernel(RowsArgs a, int rows_per_wg, int plane) {
    extern __shared__ __align__(16) float s_mem[];
    __shared__ float s_red[ROWS_WAVES];
    __shared__ float s_part[ROWS_WAVES][2];
    __shared__ int s_sel[ROWS_MAX_TOP];
    __shared__ float s_score[ROWS_MAX_TOP];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6;
    float *xs = s_mem;
    const int K = a.K, ld = a.ld;
    const int nvec = PRO == RP_DOWN ? a.top : 1;  // vectors staged, each in its own 2 * plane floats

    // the work of this wavefront: pairs of rows, each in steps of ROWS_U chunks
    const int64_t row_end = min((int64_t)(blockIdx.x + 1) * rows_per_wg, a.n_rows);
    const int pair_step = KSPLIT ? 2 : 2 * ROWS_WAVES;
    int64_t r0 = (int64_t)blockIdx.x * rows_per_wg + (KSPLIT ? 0 : 2 * wave);
    const int kw = KSPLIT ? ((ld + 511) / 512 + ROWS_WAVES - 1) / ROWS_WAVES * 512 : 0;  // inputs of a wavefront
    const int kstart = KSPLIT ? min(wave * kw, ld) : 0, kend = KSPLIT ? min(kstart + kw, ld) : ld;
    constexpr int kstep = ROWS_U * 512;
    auto row_ptrs = [&](int64_t r, int v, const uint16_t *&w0, const uint16_t *&w1) {
        const int64_t r1 = r + 1 < row_end ? r + 1 : r;
        if (PRO == RP_UP) {
            const unsigned n = (unsigned)a.rows_each, e0 = (unsigned)r / n, e1 = (unsigned)r1 / n;
            w0 = a.w + ((int64_t)s_sel[e0] * a.rows_each + (r - e0 * a.rows_each)) * ld;
            w1 = a.w + ((int64_t)s_sel[e1] * a.rows_each + (r1 - e1 * a.rows_each)) * ld;
        } else if (PRO == RP_DOWN) {
            w0 = a.w + ((int64_t)s_sel[v] * a.rows_each + r) * ld;
            w1 = a.w + ((int64_t)s_sel[v] * a.rows_each + r1) * ld;
        } else {
            w0 = a.w + r * ld;
            w1 = a.w + r1 * ld;
        }
    };
    RowsChunk cur[ROWS_U], nxt[ROWS_U];
    const uint16_t *w0 = nullptr, *w1 = nullptr;
    auto fetch = [&](RowsChunk (&c)[ROWS_U], int k) {
#pragma unroll
        for (int u = 0; u < ROWS_U; u++) rows_load(c[u], w0, w1, k + 512 * u + 8 * lane, kend);
    };
    // the first rows do not depend on the vector: they are under way while it is made
    if (PRO != RP_UP && PRO != RP_DOWN && r0 < row_end) {
        row_ptrs(r0, 0, w0, w1);
        fetch(cur, kstart);
    }

    if (PRO == RP_UP || PRO == RP_DOWN) {
        l_route(a.z, a.z_bias, a.n_experts, a.top, a.route, s_mem + (int64_t)nvec * 2 * plane, s_sel, s_score);
        if (r0 < row_end) {
            row_ptrs(r0, 0, w0, w1);
            fetch(cur, kstart);
        }
    }

    // ---- the vector -------------------------------------------------------------------------------------------
    // (four elements a thread and step; the vectors of one prologue are fetched together, ROWS_V steps at a time)
    const bool quads = K % 4 == 0 && (PRO != RP_HEADNORM || a.hv % 4 == 0);
    auto put4 = [&](float *dst, int q, float4 v) { *(float4 *)(dst + (q & 1) * plane + 4 * (q >> 1)) = v; };
    if (PRO == RP_NORM || PRO == RP_UP) {
        float r;
        if (quads && K <= 4 * ROWS_V * ROWS_THREADS) {
            float4 x[ROWS_V], w[ROWS_V];
#pragma unroll
            for (int u = 0; u < ROWS_V; u++) {
                const int i = 4 * (t + u * ROWS_THREADS);
                x[u] = w[u] = make_float4(0.f, 0.f, 0.f, 0.f);
                if (i < K) {
                    x[u] = *(const float4 *)(a.x + i);
                    w[u] = *(const float4 *)(a.normw + i);
                }
            }
            if (a.y) {
                float4 y[ROWS_V], yw[ROWS_V];
                float ss = 0.0f;
#pragma unroll
                for (int u = 0; u < ROWS_V; u++) {
                    const int i = 4 * (t + u * ROWS_THREADS);
                    y[u] = yw[u] = make_float4(0.f, 0.f, 0.f, 0.f);
                    if (i < K) {
                        y[u] = *(const float4 *)(a.y + i);
                        yw[u] = *(const float4 *)(a.yw + i);
                    }
                }
#pragma unroll
                for (int u = 0; u < ROWS_V; u++) ss = fmaf(y[u].x, y[u].x, fmaf(y[u].y, y[u].y, fmaf(y[u].z, y[u].z, fmaf(y[u].w, y[u].w, ss))));
                const float f = a.mult / sqrtf(l_block_sum(ss, s_red) / (float)K + a.eps);
#pragma unroll
                for (int u = 0; u < ROWS_V; u++) {
                    const int i = 4 * (t + u * ROWS_THREADS);
                    x[u].x = fmaf(f * y[u].x, yw[u].x, x[u].x);
                    x[u].y = fmaf(f * y[u].y, yw[u].y, x[u].y);
                    x[u].z = fmaf(f * y[u].z, yw[u].z, x[u].z);
                    x[u].w = fmaf(f * y[u].w, yw[u].w, x[u].w);
                    if (blockIdx.x == 0 && i < K) *(float4 *)(a.x_out + i) = x[u];
                }
            }
            float ss = 0.0f;
#pragma unroll
            for (int u = 0; u < ROWS_V; u++) ss = fmaf(x[u].x, x[u].x, fmaf(x[u].y, x[u].y, fmaf(x[u].z, x[u].z, fmaf(x[u].w, x[u].w, ss))));
            r = 1.0f / sqrtf(l_block_sum(ss, s_red) / (float)K + a.eps);
#pragma unroll
            for (int u = 0; u < ROWS_V; u++) {
                const int q = t + u * ROWS_THREADS;
                if (4 * q < ld) put4(xs, q, make_float4(r * x[u].x * w[u].x, r * x[u].y * w[u].y, r * x[u].z * w[u].z, r * x[u].w * w[u].w));
            }
        } else {
            float f = 0.0f;
            if (a.y) {
                float ss = 0.0f;
                for (int i = t; i < K; i += ROWS_THREADS) ss = fmaf(a.y[i], a.y[i], ss);
                f = a.mult / sqrtf(l_block_sum(ss, s_red) / (float)K + a.eps);
            }
            float ss = 0.0f;
            for (int i = t; i < ld; i += ROWS_THREADS) {
                float v = 0.0f;
                if (i < K) {
                    v = a.x[i];
                    if (a.y) {
                        v = fmaf(f * a.y[i], a.yw[i], v);
                        if (blockIdx.x == 0) a.x_out[i] = v;
                    }
                }
                ss = fmaf(v, v, ss);
                if (i < K) v *= a.normw[i];
                xs[xs_index(i, plane)] = v;
            }
            r = 1.0f / sqrtf(l_block_sum(ss, s_red) / (float)K + a.eps);
            for (int i = t; i < ld; i += ROWS_THREADS) xs[i] *= r;
        }
    } else if (PRO == RP_HEADNORM) {
        auto scale = [&](int h) {
            float ss = 0.0f;
            for (int p = 0; p < a.n_split; p++) ss += a.ssq[h * a.n_split + p];
            return 1.0f / sqrtf(ss / (float)a.hv + a.eps);
        };
        if (quads) {
            for (int q0 = t; 4 * q0 < ld; q0 += ROWS_V * ROWS_THREADS) {
                float4 x[ROWS_V], g[ROWS_V], w[ROWS_V];
                float r[ROWS_V];
#pragma unroll
                for (int u = 0; u < ROWS_V; u++) {
                    const int i = 4 * (q0 + u * ROWS_THREADS);
                    x[u] = g[u] = w[u] = make_float4(0.f, 0.f, 0.f, 0.f);
                    r[u] = 0.0f;
                    if (i < K) {
                        const int h = i / a.hv;
                        x[u] = *(const float4 *)(a.x + i);
                        g[u] = *(const float4 *)(a.gate + i);
                        w[u] = *(const float4 *)(a.normw + (i - h * a.hv));
                        r[u] = scale(h);
                    }
                }
#pragma unroll
                for (int u = 0; u < ROWS_V; u++) {
                    const int q = q0 + u * ROWS_THREADS;
                    if (4 * q < ld)
                        put4(xs, q, make_float4(r[u] * x[u].x * w[u].x * g[u].x, r[u] * x[u].y * w[u].y * g[u].y,
                                                r[u] * x[u].z * w[u].z * g[u].z, r[u] * x[u].w * w[u].w * g[u].w));
                }
            }
        } else {
            for (int i = t; i < ld; i += ROWS_THREADS) {
                float v = 0.0f;
                if (i < K) {
                    const int h = i / a.hv;
                    v = a.x[i] * scale(h) * a.normw[i - h * a.hv] * a.gate[i];
                }
                xs[xs_index(i, plane)] = v;
            }
        }
    } else {
        for (int v = 0; v < nvec; v++) {
            const float *src = a.x + (int64_t)v * K;
            float *dst = xs + v * 2 * plane;
            if (quads) {
                for (int q0 = t; 4 * q0 < ld; q0 += ROWS_V * ROWS_THREADS) {
                    float4 x[ROWS_V];
#pragma unroll
                    for (int u = 0; u < ROWS_V; u++) {
                        const int i = 4 * (q0 + u * ROWS_THREADS);
                        x[u] = i < K ? *(const float4 *)(src + i) : make_float4(0.f, 0.f, 0.f, 0.f);
                    }
#pragma unroll
                    for (int u = 0; u < ROWS_V; u++)
                        if (4 * (q0 + u * ROWS_THREADS) < ld) put4(dst, q0 + u * ROWS_THREADS, x[u]);
                }
            } else {
                for (int i = t; i < ld; i += ROWS_THREADS) dst[xs_index(i, plane)] = i < K ? src[i] : 0.0f;
            }
        }
    }
    __syncthreads();

    // ---- rows -------------------------------------------------------------------------------------------------
    int v = 0, k = kstart;
    float acc0 = 0.0f, acc1 = 0.0f;
    while (r0 < row_end) {
        // where the next step is; its chunks are fetched before this step's are used
        int64_t rn = r0;
        int vn = v, kn = k + kstep;
        if (kn >= kend) {
            kn = kstart;
            if (++vn == nvec) {
                vn = 0;
                rn = r0 + pair_step;
            }
        }
        if (rn < row_end) {
            if (rn != r0 || vn != v) row_ptrs(rn, vn, w0, w1);
            fetch(nxt, kn);
        }
        const float *xv = xs + v * 2 * plane;
#pragma unroll
        for (int u = 0; u < ROWS_U; u++) rows_fma(cur[u], xv, plane, k + 512 * u + 8 * lane, kend, acc0, acc1);
        if (rn != r0) {
            const bool two = r0 + 1 < row_end;
            acc0 = l_wave_sum(acc0);
            acc1 = l_wave_sum(acc1);
            if (KSPLIT) {
                __syncthreads();
                if (lane == 0) {
                    s_part[wave][0] = acc0;
                    s_part[wave][1] = acc1;
                }
                __syncthreads();
                acc0 = acc1 = 0.0f;
#pragma unroll
                for (int i = 0; i < ROWS_WAVES; i++) {
                    acc0 += s_part[i][0];
                    acc1 += s_part[i][1];
                }
            }
            if (EPI == RE_GLU || (EPI == RE_STORE_GLU && r0 >= a.glu_from)) {  // (whole pairs)
                if ((!KSPLIT || wave == 0) && lane == 0) {
                    float s_in = 1.0f, s_out = 1.0f;
                    if (PRO == RP_UP) (a.route == LROUTE_SIGMOID_IN ? s_in : s_out) = s_score[(unsigned)r0 / (unsigned)a.rows_each];
                    const float o = s_out * l_act(a.act, s_in * acc0) * (s_in * acc1);
                    if (EPI == RE_GLU)
                        a.out[r0 >> 1] = o;
                    else
                        a.out2[(r0 - a.glu_from) >> 1] = o;
                }
            } else if ((!KSPLIT || wave == 0) && lane < (two ? 2 : 1)) {
                const int64_t r = r0 + lane;
                const float val = lane ? acc1 : acc0;
                float o = val;
                if (EPI == RE_RESID) o = a.resid[r] + a.mult * val;
                if (EPI == RE_ACT) o = l_act(a.act, val);
                if (EPI == RE_UP) {
                    const float f = s_score[(unsigned)r / (unsigned)a.rows_each];
                    o = a.route == LROUTE_SIGMOID_IN ? l_act(a.act, f * val) : f * l_act(a.act, val);
                }
                if (EPI == RE_EMBED) o = l_act(a.act, val) * l_bf16(a.emb[(int64_t)l_step_token(a.ctl, a.prompt) * a.emb_ld + r]);
                a.out[r] = o;
            }
            acc0 = acc1 = 0.0f;
        }
#pragma unroll
        for (int u = 0; u < ROWS_U; u++) cur[u] = nxt[u];
        r0 = rn;
        v = vn;
        k = kn;
    }
}

#define ROWS_MAX_DEVICES 64

template <int PRO, int EPI, bool KSPLIT>
static hipError_t rows_launch(hipStream_t s, const RowsArgs &a, int64_t rows_per_wg) {
    const int plane = a.ld / 2;
    const int nvec = PRO == RP_DOWN ? a.top : 1;
    const size_t lds = ((size_t)nvec * 2 * plane + (PRO == RP_UP || PRO == RP_DOWN ? a.n_experts : 0)) * sizeof(float);
    if (lds > 152 * 1024) return hipErrorInvalidValue;
    if (lds > 48 * 1024) {
        int dev = 0;
        hipError_t e = hipGetDevice(&dev);
        if (e != hipSuccess) return e;
        if (dev < 0 || dev >= ROWS_MAX_DEVICES) return hipErrorInvalidDevice;
        static bool attr_set[ROWS_MAX_DEVICES] = {};
        if (!attr_set[dev]) {
            e = hipFuncSetAttribute((const void *)rows_kernel<PRO, EPI, KSPLIT>, hipFuncAttributeMaxDynamicSharedMemorySize, 152 * 1024);
            if (e != hipSuccess) return e;
            attr_set[dev] = true;
        }
    }
    const unsigned grid = (unsigned)((a.n_rows + rows_per_wg - 1) / rows_per_wg);
    hipLaunchKernelGGL((rows_kernel<PRO, EPI, KSPLIT>), dim3(grid), dim3(ROWS_THREADS), lds, s, a, (int)rows_per_wg, plane);
    return hipGetLastError();
}

template <int PRO, int EPI>
static hipError_t rows_split(hipStream_t s, const RowsArgs &a, int n_cu) {
    const int64_t pairs = (a.n_rows + 1) / 2;
    // fewer pairs of rows than wavefronts on half of the CUs: a workgroup per pair
    if (pairs < 2 * n_cu && a.ld >= 1024) return rows_launch<PRO, EPI, true>(s, a, 2);
    // about two workgroups per CU where the rows allow it; whole pairs of rows per wavefront
    int64_t per = (pairs + (int64_t)2 * n_cu - 1) / ((int64_t)2 * n_cu);
    per = (per + ROWS_WAVES - 1) / ROWS_WAVES * ROWS_WAVES;  // pairs per workgroup
    return rows_launch<PRO, EPI, false>(s, a, 2 * per);
}

hipError_t k_rows(hipStream_t s, const RowsArgs &a, int pro, int epi, int n_cu) {
    if (!a.w || !a.x || !a.out || a.n_rows < 1 || a.ld % 64 != 0 || a.K > a.ld || a.K < 1) return hipErrorInvalidValue;
    if ((pro == RP_UP || pro == RP_DOWN) &&
        (!a.z || a.n_experts < 1 || a.n_experts > ROWS_MAX_EXPERTS || a.top < 1 || a.top > ROWS_MAX_TOP || a.top > a.n_experts))
        return hipErrorInvalidValue;
    if ((epi == RE_GLU && a.n_rows % 2 != 0) || (epi == RE_STORE_GLU && (a.n_rows % 2 != 0 || a.glu_from % 2 != 0 || !a.out2)))
        return hipErrorInvalidValue;
#define GO(P, E) \
    if (pro == P && epi == E) return rows_split<P, E>(s, a, n_cu)
    GO(RP_NORM, RE_STORE);
    GO(RP_NORM, RE_ACT);
    GO(RP_PLAIN, RE_STORE);
    GO(RP_PLAIN, RE_RESID);
    GO(RP_PLAIN, RE_EMBED);
    GO(RP_UP, RE_UP);
    GO(RP_NORM, RE_GLU);
    GO(RP_NORM, RE_STORE_GLU);
    GO(RP_UP, RE_GLU);
    GO(RP_DOWN, RE_RESID);
    GO(RP_HEADNORM, RE_RESID);
#undef GO
    return hipErrorInvalidValue;
}
