// One token through a bf16 matrix: a workgroup stages the input vector in LDS behind a fused prologue (norms, expert
// choice), its wavefronts stream whole matrix rows, two at a time, 16 bytes per lane and load, and a fused epilogue writes
// the results.  Activations and sums are fp32 throughout.
#include "layered_dev.h"

#define ROWS_THREADS 256
#define ROWS_WAVES 4
#define ROWS_MAX_EXPERTS 1024
#define ROWS_MAX_TOP 64

// element e of the staged vector: the two halves of every group of 8 lie in separate planes, so that the lanes of a
// wavefront, each reading 8 consecutive elements as two 16-byte words, touch consecutive words
__device__ __forceinline__ int xs_index(int e, int plane) { return ((e >> 2) & 1) * plane + ((e >> 3) << 2) + (e & 3); }

template <int PRO, int EPI>
__global__ __launch_bounds__(ROWS_THREADS) void rows_kernel(RowsArgs a, int rows_per_wg, int plane) {
    extern __shared__ __align__(16) float s_mem[];
    __shared__ float s_red[ROWS_WAVES];
    __shared__ int s_sel[ROWS_MAX_TOP];
    __shared__ float s_score[ROWS_MAX_TOP];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6;
    float *xs = s_mem;
    const int K = a.K, ld = a.ld;
    const int nvec = PRO == RP_DOWN ? a.top : 1;  // vectors staged, each in its own 2 * plane floats

    if (PRO == RP_UP || PRO == RP_DOWN) {
        // an expert's place among all by score: the number of larger ones (the lower index first among equals)
        float *zs = s_mem + (int64_t)nvec * 2 * plane;
        for (int e = t; e < a.n_experts; e += ROWS_THREADS) zs[e] = a.z[e];
        if (t < a.top) s_sel[t] = 0, s_score[t] = 0.0f;  // (a place that no number takes, with NaN among them, stays defined)
        __syncthreads();
        for (int e = t; e < a.n_experts; e += ROWS_THREADS) {
            const float z = zs[e];
            int rank = 0;
            for (int o = 0; o < a.n_experts; o++) rank += (zs[o] > z || (zs[o] == z && o < e)) ? 1 : 0;
            if (rank < a.top) {
                s_sel[rank] = e;
                s_score[rank] = l_sigmoid(z);
            }
        }
        __syncthreads();
    }

    // ---- the vector -------------------------------------------------------------------------------------------
    if (PRO == RP_NORM || PRO == RP_UP) {
        float ry = 0.0f;
        if (a.y) {
            float ss = 0.0f;
            for (int i = t; i < K; i += ROWS_THREADS) ss = fmaf(a.y[i], a.y[i], ss);
            ry = 1.0f / sqrtf(l_block_sum(ss, s_red) / (float)K + a.eps);
        }
        float ss = 0.0f;
        for (int i = t; i < ld; i += ROWS_THREADS) {
            float v = 0.0f;
            if (i < K) {
                v = a.x[i];
                if (a.y) {
                    v += a.mult * (a.y[i] * ry * a.yw[i]);
                    if (blockIdx.x == 0) a.x_out[i] = v;
                }
            }
            xs[xs_index(i, plane)] = v;
            ss = fmaf(v, v, ss);
        }
        const float r = 1.0f / sqrtf(l_block_sum(ss, s_red) / (float)K + a.eps);
        for (int i = t; i < K; i += ROWS_THREADS) xs[xs_index(i, plane)] *= r * a.normw[i];
    } else if (PRO == RP_HEADNORM) {
        for (int i = t; i < ld; i += ROWS_THREADS) {
            float v = 0.0f;
            if (i < K) {
                const int h = i / a.hv, j = i - h * a.hv;
                float ss = 0.0f;
                for (int p = 0; p < a.n_split; p++) ss += a.ssq[h * a.n_split + p];
                v = a.x[i] / sqrtf(ss / (float)a.hv + a.eps) * a.normw[j] * a.gate[i];
            }
            xs[xs_index(i, plane)] = v;
        }
    } else {
        for (int v = 0; v < nvec; v++)
            for (int i = t; i < ld; i += ROWS_THREADS) xs[v * 2 * plane + xs_index(i, plane)] = i < K ? a.x[(int64_t)v * K + i] : 0.0f;
    }
    __syncthreads();

    // ---- rows -------------------------------------------------------------------------------------------------
    const int64_t row_end = min((int64_t)(blockIdx.x + 1) * rows_per_wg, a.n_rows);
    for (int64_t r0 = (int64_t)blockIdx.x * rows_per_wg + 2 * wave; r0 < row_end; r0 += 2 * ROWS_WAVES) {
        const bool two = r0 + 1 < row_end;
        const int64_t r1 = two ? r0 + 1 : r0;
        float acc0 = 0.0f, acc1 = 0.0f;
        for (int v = 0; v < nvec; v++) {
            const uint16_t *w0, *w1;
            if (PRO == RP_UP) {
                const int64_t e0 = r0 / a.rows_each, e1 = r1 / a.rows_each;
                w0 = a.w + ((int64_t)s_sel[e0] * a.rows_each + (r0 - e0 * a.rows_each)) * ld;
                w1 = a.w + ((int64_t)s_sel[e1] * a.rows_each + (r1 - e1 * a.rows_each)) * ld;
            } else if (PRO == RP_DOWN) {
                w0 = a.w + ((int64_t)s_sel[v] * a.rows_each + r0) * ld;
                w1 = a.w + ((int64_t)s_sel[v] * a.rows_each + r1) * ld;
            } else {
                w0 = a.w + r0 * ld;
                w1 = a.w + r1 * ld;
            }
            const float *xv = xs + v * 2 * plane;
#pragma unroll 4
            for (int k = lane * 8; k < ld; k += 512) {
                const uint4 p = *(const uint4 *)(w0 + k), q = *(const uint4 *)(w1 + k);
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
        }
        acc0 = l_wave_sum(acc0);
        acc1 = l_wave_sum(acc1);
        if (lane < (two ? 2 : 1)) {
            const int64_t r = lane ? r1 : r0;
            const float v = lane ? acc1 : acc0;
            float o = v;
            if (EPI == RE_RESID) o = a.resid[r] + a.mult * v;
            if (EPI == RE_ACT) o = l_act(a.act, v);
            if (EPI == RE_UP) o = l_act(a.act, s_score[r / a.rows_each] * v);
            if (EPI == RE_EMBED) o = l_act(a.act, v) * l_bf16(a.emb[(int64_t)l_step_token(a.ctl, a.prompt) * a.emb_ld + r]);
            a.out[r] = o;
        }
    }
}

#define ROWS_MAX_DEVICES 64

template <int PRO, int EPI>
static hipError_t rows_launch(hipStream_t s, const RowsArgs &a, int n_cu) {
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
            e = hipFuncSetAttribute((const void *)rows_kernel<PRO, EPI>, hipFuncAttributeMaxDynamicSharedMemorySize, 152 * 1024);
            if (e != hipSuccess) return e;
            attr_set[dev] = true;
        }
    }
    // about four workgroups per CU where the rows allow it; whole pairs of rows per wavefront
    const int64_t pairs = (a.n_rows + 1) / 2;
    int64_t per = (pairs + (int64_t)4 * n_cu - 1) / ((int64_t)4 * n_cu);
    per = (per + ROWS_WAVES - 1) / ROWS_WAVES * ROWS_WAVES;  // pairs per workgroup
    const int64_t rows_per_wg = 2 * per;
    const unsigned grid = (unsigned)((a.n_rows + rows_per_wg - 1) / rows_per_wg);
    hipLaunchKernelGGL((rows_kernel<PRO, EPI>), dim3(grid), dim3(ROWS_THREADS), lds, s, a, (int)rows_per_wg, plane);
    return hipGetLastError();
}

hipError_t k_rows(hipStream_t s, const RowsArgs &a, int pro, int epi, int n_cu) {
    if (!a.w || !a.x || !a.out || a.n_rows < 1 || a.ld % 64 != 0 || a.K > a.ld || a.K < 1) return hipErrorInvalidValue;
    if ((pro == RP_UP || pro == RP_DOWN) &&
        (!a.z || a.n_experts < 1 || a.n_experts > ROWS_MAX_EXPERTS || a.top < 1 || a.top > ROWS_MAX_TOP || a.top > a.n_experts))
        return hipErrorInvalidValue;
#define GO(P, E) \
    if (pro == P && epi == E) return rows_launch<P, E>(s, a, n_cu)
    GO(RP_NORM, RE_STORE);
    GO(RP_NORM, RE_ACT);
    GO(RP_PLAIN, RE_STORE);
    GO(RP_PLAIN, RE_RESID);
    GO(RP_PLAIN, RE_EMBED);
    GO(RP_UP, RE_UP);
    GO(RP_DOWN, RE_RESID);
    GO(RP_HEADNORM, RE_RESID);
#undef GO
    return hipErrorInvalidValue;
}
