// Attention over a sliding window of the last `window` positions (the query's own included), grouped heads, interleaved
// rotation and norm of q and k, one sigmoid gate per head on the output.  Keys and values are fp32 rows of a cache that is
// linear in the position: kc[G][Dp / 4][seq_len][4], vc[G][seq_len][V].
#include "layered_dev.h"

#define WIN_MAX_HEADS 8  // query heads of a key/value head handled in one pass of the one-token kernel

// ---------------------------------------------------------------------------------------------------------------
// one token: workgroup (split of the window, key/value head).  Scores: a lane holds one key of the split, the four wavefronts
// a quarter of the key elements each.  Values: groups of threads take every so-many-th key, a thread one column.
// ---------------------------------------------------------------------------------------------------------------
// NH query heads of a key/value head at a time (a missing one has a zero query)
template <int NH>
__global__ __launch_bounds__(256) void window_step_kernel(WindowShape w, const float *freq, const float *in, float *kc, float *vc,
                                                          const DecodeCtl *ctl, float *part, float *out, int n_split) {
    extern __shared__ __align__(16) float s_mem[];
    constexpr int KA = 8, VA = 32;  // key quads and value rows a thread fetches ahead
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6;
    const int g = blockIdx.y, sp = blockIdx.x, pos = ctl->pos;
    const int gq = w.H / w.G, D = w.D, Dp = w.Dp(), V = w.V, D4 = Dp / 4;
    float *s_k = s_mem, *s_q = s_k + Dp, *s_acc = s_q + NH * Dp;
    __shared__ float s_part[4][NH][L_WIN_SPLIT], s_p[NH][L_WIN_SPLIT], s_l[NH], s_m[NH];
    const int lo = max(0, pos - w.window + 1);
    const int k0 = lo + sp * L_WIN_SPLIT, n = min(L_WIN_SPLIT, pos + 1 - k0);  // this workgroup's keys
    if (n <= 0) {
        for (int i = t; i < gq; i += 256) {
            float *p = part + ((int64_t)(g * gq + i) * n_split + sp) * (V + 2);
            p[0] = -INFINITY;
            p[1] = 0.0f;
        }
        return;
    }
    const int64_t krow = (int64_t)g * D4 * w.seq_len;
    const bool has_new = k0 + n - 1 == pos;  // the token's own key and value come from its projections, not from the cache
    const int nc = has_new ? n - 1 : n;      // keys of the split that the cache holds
    const int kl = max(0, min(lane, nc - 1));  // (lanes beyond the cached keys repeat the last one)
    const int i0 = D4 * wave / 4, i1 = D4 * (wave + 1) / 4;
    const float *kp = kc + (krow + k0 + kl) * 4;
    const int tv = min(256, V), np = 256 / tv, pg = t / tv, c = t - pg * tv;  // V <= 256
    const bool mine = pg < np;
    const float *vp = vc + ((int64_t)g * w.seq_len + k0) * V + c;
    float4 kr[KA];
    float vr[VA];
#pragma unroll
    for (int u = 0; u < KA; u++) kr[u] = *(const float4 *)(kp + (int64_t)min(i0 + u, D4 - 1) * w.seq_len * 4);
#pragma unroll
    for (int u = 0; u < VA; u++) {
        const int i = pg + u * np;
        vr[u] = (mine && i < nc) ? vp[(int64_t)i * V] : 0.0f;
    }
    const float *v_new = in + w.off_v() + g * V;
    if (has_new) {
        if (wave == 3) {
            for (int i = D + lane; i < Dp; i += 64) s_k[i] = 0.0f;
            l_rotate_norm(in + w.off_k() + g * D, s_k, D, w.rot, w.rot_half, freq, pos, w.qk_norm, w.eps, lane);
        }
        for (int i = t; i < V; i += 256) vc[((int64_t)g * w.seq_len + pos) * V + i] = v_new[i];
    }
    for (int h0 = 0; h0 < gq; h0 += NH) {
        const int nh = min(NH, gq - h0);
        __syncthreads();
        for (int j = wave; j < NH; j += 4) {
            for (int i = (j < nh ? D : 0) + lane; i < Dp; i += 64) s_q[j * Dp + i] = 0.0f;
            if (j < nh) l_rotate_norm(in + (g * gq + h0 + j) * D, s_q + j * Dp, D, w.rot, w.rot_half, freq, pos, w.qk_norm, w.eps, lane);
        }
        __syncthreads();
        if (has_new && h0 == 0)
            for (int i = t; i < Dp; i += 256) kc[(krow + (int64_t)(i >> 2) * w.seq_len + pos) * 4 + (i & 3)] = s_k[i];
        float sc[NH];
#pragma unroll
        for (int j = 0; j < NH; j++) sc[j] = 0.0f;
        auto score = [&](float4 kv, int i) {
#pragma unroll
            for (int j = 0; j < NH; j++) {
                const float4 qv = *(const float4 *)(s_q + j * Dp + 4 * i);
                sc[j] = fmaf(qv.x, kv.x, sc[j]);
                sc[j] = fmaf(qv.y, kv.y, sc[j]);
                sc[j] = fmaf(qv.z, kv.z, sc[j]);
                sc[j] = fmaf(qv.w, kv.w, sc[j]);
            }
        };
#pragma unroll
        for (int u = 0; u < KA; u++)
            if (i0 + u < i1) score(kr[u], i0 + u);
        for (int i = i0 + KA; i < i1; i++) score(*(const float4 *)(kp + (int64_t)i * w.seq_len * 4), i);
#pragma unroll
        for (int j = 0; j < NH; j++) s_part[wave][j][lane] = sc[j];
        __syncthreads();
        for (int j = wave; j < nh; j += 4) {  // a wavefront per head: the whole scores, their softmax over the split
            float v = s_part[0][j][lane] + s_part[1][j][lane] + s_part[2][j][lane] + s_part[3][j][lane];
            if (has_new) {
                float own = 0.0f;
                for (int i = lane; i < D; i += 64) own = fmaf(s_q[j * Dp + i], s_k[i], own);
                own = l_wave_sum(own);
                if (lane == nc) v = own;
            }
            v = lane < n ? v * w.scale : -INFINITY;
            const float mx = wave_max_f32(v);
            const float p = lane < n ? expf(v - mx) : 0.0f;
            s_p[j][lane] = p;
            const float l = l_wave_sum(p);
            if (lane == 0) {
                s_m[j] = mx;
                s_l[j] = l;
            }
        }
        for (int j = nh + wave; j < NH; j += 4) s_p[j][lane] = 0.0f;
        __syncthreads();
        float acc[NH];
#pragma unroll
        for (int j = 0; j < NH; j++) acc[j] = 0.0f;
        if (mine) {
#pragma unroll
            for (int u = 0; u < VA; u++) {
                const int i = min(pg + u * np, L_WIN_SPLIT - 1);  // (a value past the cached keys was fetched as 0)
#pragma unroll
                for (int j = 0; j < NH; j++) acc[j] = fmaf(s_p[j][i], vr[u], acc[j]);
            }
            for (int i = pg + VA * np; i < nc; i += np) {
                const float v = vp[(int64_t)i * V];
#pragma unroll
                for (int j = 0; j < NH; j++) acc[j] = fmaf(s_p[j][i], v, acc[j]);
            }
            if (has_new && pg == 0) {
                const float v = v_new[c];
#pragma unroll
                for (int j = 0; j < NH; j++) acc[j] = fmaf(s_p[j][nc], v, acc[j]);
            }
        }
#pragma unroll
        for (int j = 0; j < NH; j++) s_acc[j * 256 + t] = acc[j];
        __syncthreads();
        for (int idx = t; idx < nh * V; idx += 256) {
            const int j = idx / V, e = idx - j * V, h = g * gq + h0 + j;
            float v = 0.0f;
            for (int p = 0; p < np; p++) v += s_acc[j * 256 + p * tv + e];
            if (n_split == 1) {
                v /= s_l[j];
                if (w.gated) v *= l_sigmoid(in[w.off_g() + h]);
                out[h * V + e] = v;
            } else {
                float *p = part + ((int64_t)h * n_split + sp) * (V + 2);
                p[2 + e] = v;
                if (e == 0) {
                    p[0] = s_m[j];
                    p[1] = s_l[j];
                }
            }
        }
    }
}

// one workgroup per head: the splits' partial results joined
__global__ __launch_bounds__(256) void window_join_kernel(WindowShape w, const float *in, const float *part, float *out, int n_split) {
    extern __shared__ __align__(16) float s_mem[];
    float *s_f = s_mem, *s_acc = s_f + n_split;
    __shared__ float s_red[4];
    const int h = blockIdx.x, V = w.V, t = threadIdx.x, st = V + 2;
    const float *p = part + (int64_t)h * n_split * st;
    float m = -INFINITY;
    for (int i = t; i < n_split; i += 256) m = fmaxf(m, p[(int64_t)i * st]);
    m = block_max_f32(m, s_red);
    float l = 0.0f;
    for (int i = t; i < n_split; i += 256) {
        const float f = expf(p[(int64_t)i * st] - m);  // (0 for a split without keys)
        s_f[i] = f;
        l = fmaf(f, p[(int64_t)i * st + 1], l);
    }
    l = l_block_sum(l, s_red);
    const float g = (w.gated ? l_sigmoid(in[w.off_g() + h]) : 1.0f) / l;
    __syncthreads();
    const int np = 256 / V, pg = t / V, c = t - pg * V;  // V <= 256
    float v = 0.0f;
    if (pg < np)
#pragma unroll 4
        for (int i = pg; i < n_split; i += np)
            if (s_f[i] != 0.0f) v = fmaf(s_f[i], p[(int64_t)i * st + 2 + c], v);
    s_acc[t] = v;
    __syncthreads();
    if (t < V) {
        v = 0.0f;
        for (int i = 0; i < np; i++) v += s_acc[i * V + t];
        out[h * V + t] = v * g;
    }
}

hipError_t k_window_step(hipStream_t s, const WindowShape &w, const float *freq, const float *in, float *kc, float *vc,
                         const DecodeCtl *ctl, float *part, float *out) {
    const int ns = window_splits(w);
    const size_t lds = (size_t)(w.Dp() * (1 + WIN_MAX_HEADS) + WIN_MAX_HEADS * 256) * sizeof(float);
    const size_t lds_join = (size_t)(ns + 256) * sizeof(float);
    if (lds > 48 * 1024 || lds_join > 60 * 1024 || w.V > 256) return hipErrorInvalidValue;
#define GO(N) \
    hipLaunchKernelGGL((window_step_kernel<N>), dim3((unsigned)ns, (unsigned)w.G), dim3(256), lds, s, w, freq, in, kc, vc, ctl, part, out, ns)
    const int gq = w.H / w.G;
    if (gq == 1)
        GO(1);
    else if (gq == 2)
        GO(2);
    else if (gq <= 4)
        GO(4);
    else
        GO(8);
#undef GO
    if (ns > 1) hipLaunchKernelGGL(window_join_kernel, dim3((unsigned)w.H), dim3(256), lds_join, s, w, in, part, out, ns);
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------------------
// many tokens
// ---------------------------------------------------------------------------------------------------------------
// one wavefront per (token, unit): units are the H query heads, then the G key/value heads
__global__ __launch_bounds__(256) void window_prepare_kernel(WindowShape w, const float *freq, const float *raw, int64_t ldr, float *kc,
                                                             float *vc, int M, int pos0, float *qf, uint16_t *qb, int hs) {
    extern __shared__ __align__(16) float s_mem[];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, D = w.D;
    const int unit = blockIdx.x * 4 + wave, m = blockIdx.y, pos = pos0 + m;
    if (unit >= w.H + w.G) return;
    float *x = s_mem + wave * D;
    const float *r = raw + (int64_t)m * ldr;
    const bool isq = unit < w.H;
    const int g = unit - w.H;
    l_rotate_norm(isq ? r + unit * D : r + w.off_k() + g * D, x, D, w.rot, w.rot_half, freq, pos, w.qk_norm, w.eps, lane);
    __builtin_amdgcn_wave_barrier();
    if (isq) {
        if (qf)
            for (int i = lane; i < D; i += 64) qf[((int64_t)m * w.H + unit) * D + i] = x[i];
        if (qb)
            for (int i = lane; i < hs; i += 64) ((__bf16 *)qb)[((int64_t)m * w.H + unit) * hs + i] = (__bf16)(i < D ? x[i] : 0.0f);
        return;
    }
    for (int i = lane; i < D; i += 64) kc[(((int64_t)g * (w.Dp() / 4) + (i >> 2)) * w.seq_len + pos) * 4 + (i & 3)] = x[i];
    for (int i = lane; i < w.V; i += 64) vc[((int64_t)g * w.seq_len + pos) * w.V + i] = r[w.off_v() + g * w.V + i];
}
hipError_t k_window_prepare(hipStream_t s, const WindowShape &w, const float *freq, const float *raw, int64_t ldr, float *kc,
                            float *vc, int M, int pos0, float *qf, uint16_t *qb, int hs) {
    if (pos0 < 0 || M < 1 || pos0 + M > w.seq_len) return hipErrorInvalidValue;
    const dim3 grid((unsigned)((w.H + w.G + 3) / 4), (unsigned)M);
    hipLaunchKernelGGL(window_prepare_kernel, grid, dim3(256), 4 * w.D * sizeof(float), s, w, freq, raw, ldr, kc, vc, M, pos0, qf, qb, hs);
    return hipGetLastError();
}

// fp32 attention: workgroup = one head x WR_Q queries, keys in tiles of WR_K; a wavefront owns WR_Q / 4 queries, its lanes
// the keys of a tile, then the value columns
#define WR_Q 16
#define WR_K 64
template <int PREC>
__global__ __launch_bounds__(256) void window_rows_kernel(WindowShape w, const float *qf, const float *raw, int64_t ldr, const float *kc,
                                                          const float *vc, int M, int pos0, void *outa, int64_t lda) {
    extern __shared__ __align__(16) float s_mem[];
    constexpr int QW = WR_Q / 4;
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6;
    const int h = blockIdx.y, q0 = blockIdx.x * WR_Q, D = w.D, Dp = w.Dp(), V = w.V, D4 = Dp / 4;
    const int g = h / (w.H / w.G);
    float *s_q = s_mem, *s_v = s_q + WR_Q * Dp, *s_p = s_v + WR_K * V;
    const int64_t krow = (int64_t)g * D4 * w.seq_len;
    for (int i = t; i < WR_Q * Dp; i += 256) {
        const int q = i / Dp, e = i - q * Dp;
        s_q[i] = (q0 + q < M && e < D) ? qf[((int64_t)(q0 + q) * w.H + h) * D + e] : 0.0f;
    }
    float mrun[QW], lrun[QW], acc[QW][4];  // V <= 256: four columns per lane
#pragma unroll
    for (int a = 0; a < QW; a++) {
        mrun[a] = -INFINITY;
        lrun[a] = 0.0f;
#pragma unroll
        for (int b = 0; b < 4; b++) acc[a][b] = 0.0f;
    }
    const int last = pos0 + min(q0 + WR_Q, M) - 1, first = max(0, pos0 + q0 - w.window + 1);
    for (int k0 = first; k0 <= last; k0 += WR_K) {
        const int n = min(WR_K, last + 1 - k0);
        __syncthreads();
        for (int i = t; i < n * V; i += 256) s_v[i] = vc[((int64_t)g * w.seq_len + k0) * V + i];
        __syncthreads();
        float sc[QW];
#pragma unroll
        for (int a = 0; a < QW; a++) sc[a] = 0.0f;
        if (lane < n)
            for (int i = 0; i < D4; i++) {
                const float4 kv = *(const float4 *)(kc + (krow + (int64_t)i * w.seq_len + k0 + lane) * 4);
#pragma unroll
                for (int a = 0; a < QW; a++) {
                    const float4 qv = *(const float4 *)(s_q + (wave * QW + a) * Dp + 4 * i);
                    sc[a] = fmaf(qv.x, kv.x, sc[a]);
                    sc[a] = fmaf(qv.y, kv.y, sc[a]);
                    sc[a] = fmaf(qv.z, kv.z, sc[a]);
                    sc[a] = fmaf(qv.w, kv.w, sc[a]);
                }
            }
#pragma unroll
        for (int a = 0; a < QW; a++) {
            const int qp = pos0 + q0 + wave * QW + a, key = k0 + lane;
            const bool see = lane < n && key <= qp && qp - key < w.window;
            const float v = see ? sc[a] * w.scale : -INFINITY;
            const float mnew = fmaxf(mrun[a], wave_max_f32(v));
            const float alpha = mnew == -INFINITY ? 1.0f : expf(mrun[a] - mnew);
            const float p = see ? expf(v - mnew) : 0.0f;
            s_p[(wave * QW + a) * WR_K + lane] = p;
            lrun[a] = lrun[a] * alpha + l_wave_sum(p);
            mrun[a] = mnew;
#pragma unroll
            for (int b = 0; b < 4; b++) acc[a][b] *= alpha;
        }
        __builtin_amdgcn_wave_barrier();
        for (int i = 0; i < n; i++)
#pragma unroll
            for (int b = 0; b < 4; b++) {
                const int c = lane + 64 * b;
                if (c < V) {
                    const float v = s_v[i * V + c];
#pragma unroll
                    for (int a = 0; a < QW; a++) acc[a][b] = fmaf(s_p[(wave * QW + a) * WR_K + i], v, acc[a][b]);
                }
            }
    }
#pragma unroll
    for (int a = 0; a < QW; a++) {
        const int m = q0 + wave * QW + a;
        if (m >= M) continue;
        float f = 1.0f / lrun[a];
        if (w.gated) f *= l_sigmoid(raw[(int64_t)m * ldr + w.off_g() + h]);
#pragma unroll
        for (int b = 0; b < 4; b++) {
            const int c = lane + 64 * b;
            if (c < V) l_store_act<PREC>(outa, m * lda + h * V + c, acc[a][b] * f);
        }
        if (h == w.H - 1)
            for (int64_t j = (int64_t)w.H * V + lane; j < lda; j += 64) l_store_act<PREC>(outa, m * lda + j, 0.0f);
    }
}
hipError_t k_window_rows(hipStream_t s, const WindowShape &w, const float *qf, const float *raw, int64_t ldr, const float *kc,
                         const float *vc, int M, int pos0, void *outa, int64_t lda, int prec) {
    if (w.V > 256 || pos0 < 0 || pos0 + M > w.seq_len) return hipErrorInvalidValue;
    const size_t lds = (size_t)(WR_Q * w.Dp() + WR_K * w.V + WR_Q * WR_K) * sizeof(float);
    if (lds > 120 * 1024) return hipErrorInvalidValue;
    const dim3 grid((unsigned)((M + WR_Q - 1) / WR_Q), (unsigned)w.H);
    const void *f = prec ? (const void *)window_rows_kernel<1> : (const void *)window_rows_kernel<0>;
    if (lds > 48 * 1024) {
        const hipError_t e = hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
    }
    if (prec)
        hipLaunchKernelGGL((window_rows_kernel<1>), grid, dim3(256), lds, s, w, qf, raw, ldr, kc, vc, M, pos0, outa, lda);
    else
        hipLaunchKernelGGL((window_rows_kernel<0>), grid, dim3(256), lds, s, w, qf, raw, ldr, kc, vc, M, pos0, outa, lda);
    return hipGetLastError();
}
