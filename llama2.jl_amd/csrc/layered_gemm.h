// Epilogues of the many-token products of layered models.
#pragma once

#include "layered_dev.h"

// results (m, L .. L + 3) of a product
template <int PREC, int EPI>
__device__ __forceinline__ void gemm_store4(const GemmArgs &a, int64_t m, int64_t L, float v0, float v1, float v2, float v3) {
    float v[4] = {v0, v1, v2, v3};
    if (EPI == GE_STORE || EPI == GE_RESID || EPI == GE_DECAY || EPI == GE_SIGMOID) {
        if (L >= a.n_rows) return;
        float *o = a.outf + m * a.ldo + L;
        // (matrices have fewer than 2^31 rows: 32-bit division)
        const unsigned h0 = EPI == GE_DECAY ? (unsigned)L / (unsigned)a.hd : 0u;
        auto value = [&](int e, float old) {
            if (EPI == GE_RESID) return fmaf(a.mult, v[e], old);
            if (EPI == GE_DECAY) return -a.rate[a.hd % 4 == 0 ? h0 : (unsigned)(L + e) / (unsigned)a.hd] * l_softplus(v[e] + a.bias[L + e]);
            if (EPI == GE_SIGMOID) return l_sigmoid(v[e]);
            return v[e];
        };
        if (a.ldo % 4 == 0 && L + 3 < a.n_rows) {
            float4 q = make_float4(0.f, 0.f, 0.f, 0.f);
            if (EPI == GE_RESID) q = *(const float4 *)o;
            *(float4 *)o = make_float4(value(0, q.x), value(1, q.y), value(2, q.z), value(3, q.w));
            return;
        }
#pragma unroll
        for (int e = 0; e < 4; e++) {
            if (L + e >= a.n_rows) break;
            o[e] = value(e, EPI == GE_RESID ? o[e] : 0.0f);
        }
    } else if (EPI == GE_GLU) {
        // (n_rows even: pairs are whole)
        const int64_t i = L >> 1;
        if (i >= a.acols) return;
        float o[2] = {0.0f, 0.0f};
        const float f = a.row_scale ? a.row_scale[m] : 1.0f, fi = a.scale_in ? f : 1.0f, fo = a.scale_in ? 1.0f : f;
#pragma unroll
        for (int e = 0; e < 2; e++)
            if (L + 2 * e < a.n_rows) o[e] = fo * l_act_rounded<PREC>(a.act, fi * v[2 * e]) * (fi * v[2 * e + 1]);
        if (PREC)
            *(float2 *)((float *)a.outa + m * a.lda + i) = make_float2(o[0], o[1]);
        else
            *(uint32_t *)((uint16_t *)a.outa + m * a.lda + i) = l_pack_bf16(o[0], o[1]);
    } else {
        if (L >= a.acols) return;  // (acols a multiple of 64: whole groups of four)
#pragma unroll
        for (int e = 0; e < 4; e++) {
            if (L + e >= a.n_rows) {
                v[e] = 0.0f;
                continue;
            }
            if (EPI == GE_UP)
                v[e] = a.scale_in ? l_act_rounded<PREC>(a.act, a.row_scale[m] * v[e]) : a.row_scale[m] * l_act_rounded<PREC>(a.act, v[e]);
            else if (EPI == GE_EMBED)
                v[e] = l_act_rounded<PREC>(a.act, v[e]) * l_bf16(a.emb[(int64_t)a.tokens[m] * a.emb_ld + L + e]);
            else
                v[e] = l_act_rounded<PREC>(a.act, v[e]);
        }
        if (PREC)
            *(float4 *)((float *)a.outa + m * a.lda + L) = make_float4(v[0], v[1], v[2], v[3]);
        else
            *(uint2 *)((uint16_t *)a.outa + m * a.lda + L) = make_uint2(l_pack_bf16(v[0], v[1]), l_pack_bf16(v[2], v[3]));
    }
}
