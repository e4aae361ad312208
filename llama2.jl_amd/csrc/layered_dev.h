// Device helpers of the layered models' kernels.
#pragma once

#include "dev_common.h"
#include "layered.h"

typedef __bf16 l_bf16x2 __attribute__((ext_vector_type(2)));

__device__ __forceinline__ uint32_t l_pack_bf16(float a, float b) {
    l_bf16x2 v;
    v.x = (__bf16)a;
    v.y = (__bf16)b;
    return __builtin_bit_cast(uint32_t, v);
}
__device__ __forceinline__ float l_bf16_lo(uint32_t w) { return __uint_as_float(w << 16); }
__device__ __forceinline__ float l_bf16_hi(uint32_t w) { return __uint_as_float(w & 0xFFFF0000u); }
__device__ __forceinline__ float l_bf16(uint16_t w) { return __uint_as_float((uint32_t)w << 16); }

__device__ __forceinline__ float l_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float l_silu(float z) { return z / (1.0f + expf(-z)); }
// log(1 + exp(z)) = max(z, 0) + log(1 + e), e = exp(-|z|); log(1 + e) = 2 artanh(s), s = e / (2 + e) <= 1/3, by its power series
// (the first term left out is 2 s^17 / 17 < 1e-9 of the sum): small relative error also where the result is small
__device__ __forceinline__ float l_softplus(float z) {
    const float e = expf(-fabsf(z)), s = e / (2.0f + e), q = s * s;
    float p = fmaf(q, 1.0f / 15.0f, 1.0f / 13.0f);
    p = fmaf(p, q, 1.0f / 11.0f);
    p = fmaf(p, q, 1.0f / 9.0f);
    p = fmaf(p, q, 1.0f / 7.0f);
    p = fmaf(p, q, 1.0f / 5.0f);
    p = fmaf(p, q, 1.0f / 3.0f);
    p = fmaf(p, q, 1.0f);
    return fmaf(2.0f * s, p, fmaxf(z, 0.0f));
}
__device__ __forceinline__ float l_act(int act, float z) {
    if (act == LACT_RELU2) {
        const float r = fmaxf(z, 0.0f);
        return r * r;
    }
    if (act == LACT_RELU) return fmaxf(z, 0.0f);
    if (act == LACT_SILU) return l_silu(z);
    if (act == LACT_GELU_TANH) return 0.5f * z * (1.0f + tanhf(0.797884560802865356f * fmaf(0.044715f * z * z, z, z)));
    return 0.5f * z * (1.0f + erff(z * 0.707106781186547524f));
}
// erf by formula 7.1.26 of Abramowitz and Stegun, Handbook of Mathematical Functions: within 1.5e-7 everywhere, a dozen
// instructions; for results that are rounded to bf16
__device__ __forceinline__ float l_erf_short(float x) {
    const float a = fabsf(x), t = __builtin_amdgcn_rcpf(fmaf(0.3275911f, a, 1.0f));
    float p = fmaf(1.061405429f, t, -1.453152027f);
    p = fmaf(p, t, 1.421413741f);
    p = fmaf(p, t, -0.284496736f);
    p = fmaf(p, t, 0.254829592f);
    return copysignf(1.0f - p * t * __builtin_amdgcn_exp2f(-1.44269504088896341f * a * a), x);
}
// the activation of a result of the given precision
template <int PREC>
__device__ __forceinline__ float l_act_rounded(int act, float z) {
    if (PREC == 0 && act == LACT_GELU_ERF) return 0.5f * z * (1.0f + l_erf_short(z * 0.707106781186547524f));
    return l_act(act, z);
}

__device__ __forceinline__ float l_wave_sum(float v) {
#pragma unroll
    for (int m = 32; m >= 1; m >>= 1) v += __shfl_xor(v, m, WAVE);
    return v;
}
// sum over the workgroup; `red` holds one float per wavefront; every thread gets the total
__device__ __forceinline__ float l_block_sum(float v, float *red) {
    const int nw = (blockDim.x + 63) >> 6;
    v = l_wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    float t = 0.0f;
    for (int w = 0; w < nw; w++) t += red[w];
    return t;
}

// activations: bf16 or fp32 elements behind one pointer
template <int PREC>
__device__ __forceinline__ void l_store_act(void *p, int64_t i, float v) {
    if (PREC)
        ((float *)p)[i] = v;
    else
        ((__bf16 *)p)[i] = (__bf16)v;
}

// the token of the current decode step (as embed_kernel picks it)
__device__ __forceinline__ int l_step_token(const DecodeCtl *ctl, const int32_t *prompt) {
    return ctl->step < ctl->n_prompt ? prompt[ctl->step] : ctl->last_argmax;
}

// Rotation of the pairs (2 i, 2 i + 1), or with `half` (i, i + rot / 2), i < rot / 2, of one head at `pos` and division by the
// head's root mean square, by one wavefront.  src and dst hold D elements.
__device__ __forceinline__ void l_rotate_norm(const float *src, float *dst, int D, int rot, int half, const float *freq, int pos,
                                              int norm, float eps, int lane) {
    float ss = 0.0f;
    for (int p = lane; 2 * p < D; p += 64) {
        const bool turned = 2 * p < rot, apart = half && turned;
        const int ia = apart ? p : 2 * p, ib = apart ? p + rot / 2 : 2 * p + 1;
        float a = src[ia], b = ib < D ? src[ib] : 0.0f;
        if (turned) {
            const float ang = (float)pos * freq[p];
            const float c = cosf(ang), s = sinf(ang), u = a, v = b;
            a = u * c - v * s;
            b = v * c + u * s;
        }
        ss = fmaf(a, a, ss);
        ss = fmaf(b, b, ss);
        dst[ia] = a;
        if (ib < D) dst[ib] = b;
    }
    if (!norm) return;
    const float r = 1.0f / sqrtf(l_wave_sum(ss) / (float)D + eps);
    for (int p = lane; 2 * p < D; p += 64) {
        const bool apart = half && 2 * p < rot;
        const int ia = apart ? p : 2 * p, ib = apart ? p + rot / 2 : 2 * p + 1;
        dst[ia] *= r;
        if (ib < D) dst[ib] *= r;
    }
}

// Choice of experts by one workgroup: an expert's place among all by its logit is the number of larger ones (the lower index
// first among equals); sel[place], score[place] for the first `top` places.  zs: LDS for E logits; sel and score are LDS or
// global memory of the workgroup's own.
__device__ __forceinline__ void l_route(const float *z, const float *bias, int E, int top, int kind, float *zs, int *sel, float *score) {
    const int t = threadIdx.x, nt = blockDim.x;
    for (int e = t; e < E; e += nt) zs[e] = z[e] + (bias ? bias[e] : 0.0f);
    for (int k = t; k < top; k += nt) sel[k] = 0, score[k] = 0.0f;  // (a place that no number takes, with NaN among them, stays defined)
    __syncthreads();
    for (int e = t; e < E; e += nt) {
        const float v = zs[e];
        int rank = 0;
#pragma unroll 8
        for (int o = 0; o < E; o++) rank += (zs[o] > v || (zs[o] == v && o < e)) ? 1 : 0;
        if (rank < top) {
            sel[rank] = e;
            score[rank] = kind == LROUTE_SIGMOID_IN ? l_sigmoid(v) : v;
        }
    }
    __syncthreads();
    if (kind == LROUTE_SOFTMAX_OUT) {
        if (t < 64) {  // (top <= 64)
            const float v = t < top ? score[t] : -INFINITY, m = wave_max_f32(v);
            const float p = t < top ? expf(v - m) : 0.0f, sum = l_wave_sum(p);
            if (t < top) score[t] = p / sum;
        }
        __syncthreads();
    }
}
