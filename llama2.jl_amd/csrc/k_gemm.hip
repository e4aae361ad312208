// Many tokens through a bf16 matrix, C[m][n] = sum_k X[m][k] W[n][k], on the matrix cores: bf16 activations
// (v_mfma_f32_32x32x16_bf16) or fp32 ones (v_mfma_f32_32x32x2_f32: fp32 operands and sums), with fused epilogues and a grouped
// form for mixtures of experts; and the row-wise kernels around the products.
#include "layered_gemm.h"

typedef __bf16 l_bf16x8 __attribute__((ext_vector_type(8)));
typedef float l_f32x16 __attribute__((ext_vector_type(16)));

// Placement of the 16-byte chunks of a 128-byte tile row: 16 consecutive rows' chunks of one index fall into different slots
// of the 256-byte bank row.
__device__ __forceinline__ int gemm_swz(int r) { return (r >> 1) & 7; }

template <int PREC, int EPI, int TN, int TM, bool GROUPED>
__global__ __launch_bounds__(256) void gemm_kernel(GemmArgs a) {
    constexpr int IN = TN / 64, JM = TM / 64;          // 32 x 32 tiles per wavefront (2 x 2 wavefronts)
    constexpr int KSTEP = PREC ? 32 : 64;
    constexpr int FROW = 33;                            // floats per LDS row of the fp32 form
    __shared__ __align__(16) unsigned char s_raw[(TN + TM) * (PREC ? FROW * 4 : 128)];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6, wn = wave & 1, wm = wave >> 1;
    const uint16_t *W = a.w;
    int64_t mb = 0;
    int mcount = a.M;
    const int64_t n0 = (int64_t)blockIdx.y * TN;
    int m0 = blockIdx.x * TM;
    if (GROUPED) {
        if ((int)blockIdx.x >= a.n_tiles[0]) return;
        const GemmTile gt = a.tiles[blockIdx.x];
        W += gt.expert * a.expert_stride;
        mb = gt.row0;
        mcount = gt.n;
        m0 = 0;
    }
    l_f32x16 acc[IN][JM];
#pragma unroll
    for (int i = 0; i < IN; i++)
#pragma unroll
        for (int j = 0; j < JM; j++)
#pragma unroll
            for (int r = 0; r < 16; r++) acc[i][j][r] = 0.0f;

    // rows this thread copies: row t / 8 + 32 i of each tile, elements 8 (t % 8) .. (bf16) or 4 (t % 8) .. (fp32) of a step
    constexpr int WL = TN / 32, XL = TM / 32;
    const int c8 = t & 7;
    const uint16_t *wrow[WL];
    const uint16_t *xrow16[XL];
    const float *xrow32[XL];
#pragma unroll
    for (int i = 0; i < WL; i++) {
        int64_t r = n0 + (t >> 3) + 32 * i;
        if (r >= a.n_rows) r = a.n_rows - 1;
        wrow[i] = W + r * a.ld + (PREC ? 4 : 8) * c8;
    }
#pragma unroll
    for (int i = 0; i < XL; i++) {
        int m = m0 + (t >> 3) + 32 * i;
        if (m >= mcount) m = mcount - 1;  // (repeats the last row; not stored)
        int64_t row = mb + m;
        if (a.gather) row = a.gather[row];
        if (PREC)
            xrow32[i] = (const float *)a.x + row * a.ldx + 4 * c8;
        else
            xrow16[i] = (const uint16_t *)a.x + row * a.ldx + 8 * c8;
    }
    uint4 wreg[WL], xreg[XL];
    auto gload = [&](int k0) {
#pragma unroll
        for (int i = 0; i < WL; i++) {
            if (PREC) {
                const uint2 v = *(const uint2 *)(wrow[i] + k0);
                wreg[i] = make_uint4(v.x, v.y, 0, 0);
            } else {
                wreg[i] = *(const uint4 *)(wrow[i] + k0);
            }
        }
#pragma unroll
        for (int i = 0; i < XL; i++) xreg[i] = PREC ? *(const uint4 *)(xrow32[i] + k0) : *(const uint4 *)(xrow16[i] + k0);
    };
    gload(0);
    for (int k0 = 0; k0 < a.ld; k0 += KSTEP) {
        if constexpr (PREC == 0) {
            uint4 *s_w = (uint4 *)s_raw, *s_x = s_w + TN * 8;
#pragma unroll
            for (int i = 0; i < WL; i++) {
                const int r = (t >> 3) + 32 * i;
                s_w[r * 8 + (c8 ^ gemm_swz(r))] = wreg[i];
            }
#pragma unroll
            for (int i = 0; i < XL; i++) {
                const int r = (t >> 3) + 32 * i;
                s_x[r * 8 + (c8 ^ gemm_swz(r))] = xreg[i];
            }
            __syncthreads();
            if (k0 + KSTEP < a.ld) gload(k0 + KSTEP);
#pragma unroll
            for (int kk = 0; kk < 4; kk++) {
                const int c = 2 * kk + (lane >> 5);
                l_bf16x8 A[IN], B[JM];
#pragma unroll
                for (int i = 0; i < IN; i++) {
                    const int r = (TN / 2) * wn + 32 * i + (lane & 31);
                    A[i] = __builtin_bit_cast(l_bf16x8, s_w[r * 8 + (c ^ gemm_swz(r))]);
                }
#pragma unroll
                for (int j = 0; j < JM; j++) {
                    const int r = (TM / 2) * wm + 32 * j + (lane & 31);
                    B[j] = __builtin_bit_cast(l_bf16x8, s_x[r * 8 + (c ^ gemm_swz(r))]);
                }
#pragma unroll
                for (int i = 0; i < IN; i++)
#pragma unroll
                    for (int j = 0; j < JM; j++) acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(A[i], B[j], acc[i][j], 0, 0, 0);
            }
        } else {
            float *s_w = (float *)s_raw, *s_x = s_w + TN * FROW;
#pragma unroll
            for (int i = 0; i < WL; i++) {
                float *p = s_w + ((t >> 3) + 32 * i) * FROW + 4 * c8;
                p[0] = l_bf16_lo(wreg[i].x);
                p[1] = l_bf16_hi(wreg[i].x);
                p[2] = l_bf16_lo(wreg[i].y);
                p[3] = l_bf16_hi(wreg[i].y);
            }
#pragma unroll
            for (int i = 0; i < XL; i++) {
                float *p = s_x + ((t >> 3) + 32 * i) * FROW + 4 * c8;
                p[0] = __uint_as_float(xreg[i].x);
                p[1] = __uint_as_float(xreg[i].y);
                p[2] = __uint_as_float(xreg[i].z);
                p[3] = __uint_as_float(xreg[i].w);
            }
            __syncthreads();
            if (k0 + KSTEP < a.ld) gload(k0 + KSTEP);
#pragma unroll 4
            for (int kk = 0; kk < KSTEP; kk += 2) {
                const int c = kk + (lane >> 5);
                float A[IN], B[JM];
#pragma unroll
                for (int i = 0; i < IN; i++) A[i] = s_w[((TN / 2) * wn + 32 * i + (lane & 31)) * FROW + c];
#pragma unroll
                for (int j = 0; j < JM; j++) B[j] = s_x[((TM / 2) * wm + 32 * j + (lane & 31)) * FROW + c];
#pragma unroll
                for (int i = 0; i < IN; i++)
#pragma unroll
                    for (int j = 0; j < JM; j++) acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x2f32(A[i], B[j], acc[i][j], 0, 0, 0);
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int j = 0; j < JM; j++) {
        const int m = m0 + (TM / 2) * wm + 32 * j + (lane & 31);
        if (m >= mcount) continue;
#pragma unroll
        for (int i = 0; i < IN; i++)
#pragma unroll
            for (int rq = 0; rq < 4; rq++)
                gemm_store4<PREC, EPI>(a, mb + m, n0 + (TN / 2) * wn + 32 * i + 8 * rq + 4 * (lane >> 5), acc[i][j][4 * rq],
                                       acc[i][j][4 * rq + 1], acc[i][j][4 * rq + 2], acc[i][j][4 * rq + 3]);
    }
}

template <int PREC, int EPI>
static hipError_t gemm_launch(hipStream_t s, const GemmArgs &a) {
    // columns the epilogue covers: an activation-typed result is zeroed up to its row stride
    const bool acts = EPI == GE_ACT || EPI == GE_UP || EPI == GE_EMBED;
    const int64_t cols = EPI == GE_GLU ? 2 * a.acols : acts ? a.acols : a.n_rows;
    if (a.tiles) {
        if (EPI != GE_STORE && EPI != GE_UP && EPI != GE_GLU) return hipErrorInvalidValue;
        constexpr int E = EPI == GE_UP || EPI == GE_GLU ? EPI : GE_STORE;
        if (cols > 64) {
            hipLaunchKernelGGL((gemm_kernel<PREC, E, 128, L_GEMM_TILE, true>), dim3((unsigned)a.max_tiles, (unsigned)((cols + 127) / 128)),
                               dim3(256), 0, s, a);
        } else {
            hipLaunchKernelGGL((gemm_kernel<PREC, E, 64, L_GEMM_TILE, true>), dim3((unsigned)a.max_tiles, (unsigned)((cols + 63) / 64)),
                               dim3(256), 0, s, a);
        }
        return hipGetLastError();
    }
    const int64_t big = ((cols + 127) / 128) * ((a.M + 127) / 128);
    if (big >= 256)
        hipLaunchKernelGGL((gemm_kernel<PREC, EPI, 128, 128, false>), dim3((unsigned)((a.M + 127) / 128), (unsigned)((cols + 127) / 128)),
                           dim3(256), 0, s, a);
    else
        hipLaunchKernelGGL((gemm_kernel<PREC, EPI, 64, 64, false>), dim3((unsigned)((a.M + 63) / 64), (unsigned)((cols + 63) / 64)),
                           dim3(256), 0, s, a);
    return hipGetLastError();
}

hipError_t k_gemm(hipStream_t s, const GemmArgs &args, int prec, int epi) {
    GemmArgs a = args;
    if (!a.acols) a.acols = a.lda;
    if (!a.w || !a.x || a.n_rows < 1 || a.M < 1 || a.ld % 64 != 0 || a.ldx < a.ld || a.lda % 64 != 0 || a.acols % 64 != 0 ||
        a.acols > a.lda)
        return hipErrorInvalidValue;
    const bool acts = epi == GE_ACT || epi == GE_UP || epi == GE_EMBED;
    if (epi == GE_GLU ? (!a.outa || a.n_rows % 2 != 0 || 2 * a.acols < a.n_rows)
        : acts        ? (!a.outa || a.acols < a.n_rows)
                      : (!a.outf || a.ldo < a.n_rows))
        return hipErrorInvalidValue;
#define GO(E) \
    case E: return prec ? gemm_launch<1, E>(s, a) : gemm_launch<0, E>(s, a)
    switch (epi) {
        GO(GE_STORE);
        GO(GE_RESID);
        GO(GE_ACT);
        GO(GE_UP);
        GO(GE_EMBED);
        GO(GE_DECAY);
        GO(GE_SIGMOID);
        GO(GE_GLU);
    }
#undef GO
    return hipErrorInvalidValue;
}

// ---------------------------------------------------------------------------------------------------------------
// rows: pending update, norm, conversion to activations
// ---------------------------------------------------------------------------------------------------------------
// NQ: quads of elements a thread holds (K a multiple of 4, at most 1024 NQ); 0: any K, element by element
template <int PREC, int NQ>
__global__ __launch_bounds__(256) void norm_rows_kernel(float *X, int K, const float *w, float eps, const float *Y, const float *yw,
                                                        float mult, const int32_t *gather, void *outa, int64_t lda) {
    __shared__ float s_red[4];
    const int64_t m = blockIdx.x, src = gather ? gather[m] : m;
    float *x = X + src * K;
    const float *y = Y ? Y + src * K : nullptr;
    const int t = threadIdx.x;
    if constexpr (NQ > 0) {
        float4 v[NQ];
#pragma unroll
        for (int u = 0; u < NQ; u++) {
            const int i = 4 * (t + 256 * u);
            v[u] = i < K ? *(const float4 *)(x + i) : make_float4(0.f, 0.f, 0.f, 0.f);
        }
        if (y) {
            float4 z[NQ];
            float ss = 0.0f;
#pragma unroll
            for (int u = 0; u < NQ; u++) {
                const int i = 4 * (t + 256 * u);
                z[u] = i < K ? *(const float4 *)(y + i) : make_float4(0.f, 0.f, 0.f, 0.f);
                ss = fmaf(z[u].x, z[u].x, fmaf(z[u].y, z[u].y, fmaf(z[u].z, z[u].z, fmaf(z[u].w, z[u].w, ss))));
            }
            const float f = mult / sqrtf(l_block_sum(ss, s_red) / (float)K + eps);
#pragma unroll
            for (int u = 0; u < NQ; u++) {
                const int i = 4 * (t + 256 * u);
                if (i >= K) continue;
                const float4 g = *(const float4 *)(yw + i);
                v[u].x = fmaf(f * z[u].x, g.x, v[u].x);
                v[u].y = fmaf(f * z[u].y, g.y, v[u].y);
                v[u].z = fmaf(f * z[u].z, g.z, v[u].z);
                v[u].w = fmaf(f * z[u].w, g.w, v[u].w);
                *(float4 *)(x + i) = v[u];
            }
        }
        float r = 1.0f;
        if (w) {
            float ss = 0.0f;
#pragma unroll
            for (int u = 0; u < NQ; u++) ss = fmaf(v[u].x, v[u].x, fmaf(v[u].y, v[u].y, fmaf(v[u].z, v[u].z, fmaf(v[u].w, v[u].w, ss))));
            r = 1.0f / sqrtf(l_block_sum(ss, s_red) / (float)K + eps);
        }
        if (!outa) return;
#pragma unroll
        for (int u = 0; u < NQ; u++) {
            const int i = 4 * (t + 256 * u);
            if (i >= lda) continue;
            const float4 g = w && i < K ? *(const float4 *)(w + i) : make_float4(1.f, 1.f, 1.f, 1.f);
            const float4 q = make_float4(v[u].x * r * g.x, v[u].y * r * g.y, v[u].z * r * g.z, v[u].w * r * g.w);
            if (PREC)
                *(float4 *)((float *)outa + m * lda + i) = q;
            else
                *(uint2 *)((uint16_t *)outa + m * lda + i) = make_uint2(l_pack_bf16(q.x, q.y), l_pack_bf16(q.z, q.w));
        }
        return;
    }
    float ry = 0.0f;
    if (y) {
        float ss = 0.0f;
        for (int i = t; i < K; i += 256) ss = fmaf(y[i], y[i], ss);
        ry = 1.0f / sqrtf(l_block_sum(ss, s_red) / (float)K + eps);
    }
    float r = 1.0f;
    if (w || y) {
        float ss = 0.0f;
        for (int i = t; i < K; i += 256) {
            float v = x[i];
            if (y) {
                v += mult * (y[i] * ry * yw[i]);
                x[i] = v;
            }
            ss = fmaf(v, v, ss);
        }
        if (w) r = 1.0f / sqrtf(l_block_sum(ss, s_red) / (float)K + eps);
    }
    if (!outa) return;
    for (int64_t i = t; i < lda; i += 256) {
        float v = 0.0f;
        if (i < K) v = w ? x[i] * r * w[i] : x[i];
        l_store_act<PREC>(outa, m * lda + i, v);
    }
}
hipError_t k_norm_rows(hipStream_t s, float *x, int K, int M, const float *w, float eps, const float *y, const float *yw,
                       float mult, const int32_t *gather, void *outa, int64_t lda, int prec) {
    if (M < 1 || (y && gather)) return hipErrorInvalidValue;
#define GO(N)                                                                                                                             \
    do {                                                                                                                                  \
        if (prec)                                                                                                                         \
            hipLaunchKernelGGL((norm_rows_kernel<1, N>), dim3((unsigned)M), dim3(256), 0, s, x, K, w, eps, y, yw, mult, gather, outa, lda); \
        else                                                                                                                              \
            hipLaunchKernelGGL((norm_rows_kernel<0, N>), dim3((unsigned)M), dim3(256), 0, s, x, K, w, eps, y, yw, mult, gather, outa, lda); \
    } while (0)
    // (lda, a multiple of 64, may exceed K by up to 63 columns: they are covered, too)
    const int64_t cols = std::max<int64_t>(K, outa ? lda : 0);
    if (K % 4 != 0 || cols > 8192)
        GO(0);
    else if (cols <= 1024)
        GO(1);
    else if (cols <= 2048)
        GO(2);
    else if (cols <= 4096)
        GO(4);
    else
        GO(8);
#undef GO
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------------------
// mixture of experts
// ---------------------------------------------------------------------------------------------------------------
// one workgroup per token
__global__ __launch_bounds__(64) void route_kernel(const float *z, int64_t ldz, const float *bias, int E, int top, int kind, int32_t *choice,
                                                   float *score) {
    extern __shared__ __align__(16) float s_mem[];
    __shared__ int s_sel[64];
    __shared__ float s_score[64];
    const int64_t m = blockIdx.x;
    l_route(z + m * ldz, bias, E, top, kind, s_mem, s_sel, s_score);
    for (int k = threadIdx.x; k < top; k += 64) {
        choice[m * top + k] = s_sel[k];
        score[m * top + k] = s_score[k];
    }
}
hipError_t k_route(hipStream_t s, const float *z, int64_t ldz, const float *bias, int M, int E, int top, int kind, int32_t *choice,
                   float *score) {
    if (E < 1 || top < 1 || top > E || top > 64) return hipErrorInvalidValue;
    hipLaunchKernelGGL(route_kernel, dim3((unsigned)M), dim3(64), E * sizeof(float), s, z, ldz, bias, E, top, kind, choice, score);
    return hipGetLastError();
}

// one workgroup: counts, offsets, slots and the list of tiles.  The order of an expert's slots is whatever the LDS counters
// give; every slot is computed on its own, so no result depends on it.
__global__ __launch_bounds__(1024) void group_kernel(const int32_t *choice, const float *score, int M, int E, int top, int32_t *slot_row,
                                                     float *slot_scale, int32_t *slot_of, GemmTile *tiles, int32_t *n_tiles, int tile_rows) {
    extern __shared__ __align__(16) int s_int[];
    int *cnt = s_int, *off = s_int + E;
    const int n = M * top;
    for (int e = threadIdx.x; e < E; e += 1024) cnt[e] = 0;
    __syncthreads();
    for (int i = threadIdx.x; i < n; i += 1024) atomicAdd(&cnt[choice[i]], 1);
    __syncthreads();
    if (threadIdx.x == 0) {
        int o = 0, nt = 0;
        for (int e = 0; e < E; e++) {
            off[e] = o;
            for (int r = 0; r < cnt[e]; r += tile_rows) tiles[nt++] = GemmTile{e, o + r, min(tile_rows, cnt[e] - r)};
            o += cnt[e];
        }
        n_tiles[0] = nt;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < n; i += 1024) {
        const int slot = atomicAdd(&off[choice[i]], 1);
        slot_row[slot] = i / top;
        slot_scale[slot] = score[i];
        slot_of[i] = slot;
    }
}
hipError_t k_group(hipStream_t s, const int32_t *choice, const float *score, int M, int E, int top, int32_t *slot_row,
                   float *slot_scale, int32_t *slot_of, GemmTile *tiles, int32_t *n_tiles, int tile_rows) {
    hipLaunchKernelGGL(group_kernel, dim3(1), dim3(1024), 2 * E * sizeof(int), s, choice, score, M, E, top, slot_row, slot_scale, slot_of,
                       tiles, n_tiles, tile_rows);
    return hipGetLastError();
}

__global__ __launch_bounds__(256) void gather_add_kernel(float *x, const float *y, const int32_t *slot_of, int top, int K, float mult) {
    const int64_t m = blockIdx.y;
    const int i = 4 * (blockIdx.x * 256 + threadIdx.x);
    if (i >= K) return;
    if (K % 4 == 0) {
        const float4 a = *(const float4 *)(x + m * K + i);
        float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll 4
        for (int k = 0; k < top; k++) {
            const float4 q = *(const float4 *)(y + (int64_t)slot_of[m * top + k] * K + i);
            v.x += q.x;
            v.y += q.y;
            v.z += q.z;
            v.w += q.w;
        }
        *(float4 *)(x + m * K + i) = make_float4(fmaf(mult, v.x, a.x), fmaf(mult, v.y, a.y), fmaf(mult, v.z, a.z), fmaf(mult, v.w, a.w));
        return;
    }
    for (int e = i; e < min(i + 4, K); e++) {
        float v = 0.0f;
        for (int k = 0; k < top; k++) v += y[(int64_t)slot_of[m * top + k] * K + e];
        x[m * K + e] = fmaf(mult, v, x[m * K + e]);
    }
}
hipError_t k_gather_add(hipStream_t s, float *x, const float *y, const int32_t *slot_of, int M, int top, int K, float mult) {
    hipLaunchKernelGGL(gather_add_kernel, dim3((unsigned)((K + 1023) / 1024), (unsigned)M), dim3(256), 0, s, x, y, slot_of, top, K, mult);
    return hipGetLastError();
}

__global__ __launch_bounds__(256) void stream_add_kernel(float *x, const float *a, const float *b, int K) {
    const int i = blockIdx.x * 256 + threadIdx.x;
    if (i >= K) return;
    const int64_t at = (int64_t)blockIdx.y * K + i;
    x[at] = (a ? x[at] + a[at] : x[at]) + b[i];
}
hipError_t k_stream_add(hipStream_t s, float *x, const float *a, const float *b, int M, int K) {
    hipLaunchKernelGGL(stream_add_kernel, dim3((unsigned)((K + 255) / 256), (unsigned)M), dim3(256), 0, s, x, a, b, K);
    return hipGetLastError();
}

template <int PREC>
__global__ __launch_bounds__(256) void embed_rows_kernel(const float *v, int N, int act, const uint16_t *emb, int64_t emb_ld,
                                                         const int32_t *tokens, void *outa, int64_t lda) {
    const int64_t m = blockIdx.y;
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= lda) return;
    l_store_act<PREC>(outa, m * lda + i, i < N ? l_act(act, v[m * N + i]) * l_bf16(emb[(int64_t)tokens[m] * emb_ld + i]) : 0.0f);
}
hipError_t k_embed_rows(hipStream_t s, const float *v, int M, int N, int act, const uint16_t *emb, int64_t emb_ld,
                        const int32_t *tokens, void *outa, int64_t lda, int prec) {
    const dim3 grid((unsigned)((lda + 255) / 256), (unsigned)M);
    if (prec)
        hipLaunchKernelGGL((embed_rows_kernel<1>), grid, dim3(256), 0, s, v, N, act, emb, emb_ld, tokens, outa, lda);
    else
        hipLaunchKernelGGL((embed_rows_kernel<0>), grid, dim3(256), 0, s, v, N, act, emb, emb_ld, tokens, outa, lda);
    return hipGetLastError();
}
