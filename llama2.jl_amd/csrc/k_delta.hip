// Gated delta rule with one decay per head and key channel.  Per head, with state S [D][V] (fp32), unit vectors q and k,
// decay g [D], step size beta:
//   S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q = (decayed S)^T q + (k . q) u
// so both products of a token are taken of the decayed state, before its own write.
// The value columns of S are independent of one another: workgroups split them.
#include "layered_dev.h"

// ---------------------------------------------------------------------------------------------------------------
// one token: workgroup (split, head), 32 value columns x 8 groups of key channels
// ---------------------------------------------------------------------------------------------------------------
#define CONV_AHEAD 4  // taps whose inputs are fetched together

// the channel's convolution at `pos`: cur is its projection, ring slot `now` = pos % taps will hold it
__device__ __forceinline__ float delta_conv(const float *conv, const float *ring, int C, int taps, float cur, int ch, int pos, int now) {
    float w[CONV_AHEAD], x[CONV_AHEAD];
#pragma unroll
    for (int j = 0; j < CONV_AHEAD; j++) {
        const bool use = j < taps && j <= pos;
        const int slot = now - j < 0 ? now - j + taps : now - j;
        w[j] = use ? conv[(int64_t)(taps - 1 - j) * C + ch] : 0.0f;
        x[j] = j == 0 ? cur : use ? ring[(int64_t)slot * C + ch] : 0.0f;
    }
    float v = 0.0f;
#pragma unroll
    for (int j = 0; j < CONV_AHEAD; j++) v = fmaf(w[j], x[j], v);
    for (int j = CONV_AHEAD; j < taps && j <= pos; j++)
        v = fmaf(conv[(int64_t)(taps - 1 - j) * C + ch], ring[(int64_t)((pos - j) % taps) * C + ch], v);
    return l_silu(v);
}

// 8 lanes take a bf16 row (zero-padded to ld) against a vector in LDS; every one of them gets the sum
__device__ __forceinline__ float delta_fma8(uint4 p, const float *x, float acc) {
    const float4 a = *(const float4 *)x, b = *(const float4 *)(x + 4);
    acc = fmaf(l_bf16_lo(p.x), a.x, acc);
    acc = fmaf(l_bf16_hi(p.x), a.y, acc);
    acc = fmaf(l_bf16_lo(p.y), a.z, acc);
    acc = fmaf(l_bf16_hi(p.y), a.w, acc);
    acc = fmaf(l_bf16_lo(p.z), b.x, acc);
    acc = fmaf(l_bf16_hi(p.z), b.y, acc);
    acc = fmaf(l_bf16_lo(p.w), b.z, acc);
    return fmaf(l_bf16_hi(p.w), b.w, acc);
}
__device__ __forceinline__ float delta_sum8(float acc) {
#pragma unroll
    for (int m = 4; m >= 1; m >>= 1) acc += __shfl_xor(acc, m, WAVE);
    return acc;
}

// NR: rows of S per thread (D <= 8 NR)
template <int NR>
__global__ __launch_bounds__(256) void delta_step_kernel(DeltaShape d, DeltaWeights w, const float *in, float *ring, float *state,
                                                         const DecodeCtl *ctl, float *o, float *ssq, float *gate, int n_split) {
    extern __shared__ __align__(16) float s_mem[];
    float *s_q = s_mem, *s_k = s_q + 8 * NR, *s_g = s_k + 8 * NR, *s_fa = s_g + 8 * NR, *s_fg = s_fa + w.lda2;
    __shared__ float s_v[L_DELTA_COLS], s_red[2][8][L_DELTA_COLS], s_kq;
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6;
    const int sp = blockIdx.x, h = blockIdx.y, kvh = h / (d.H / d.G), pos = ctl->pos;
    const int D = d.D, V = d.V, c0 = sp * L_DELTA_COLS, GD = d.G * D;
    const int col = t & 31, rg = t >> 5, c = c0 + col;
    const bool live = c < V;
    float *S = state + (int64_t)h * D * V;
    float s[NR];
#pragma unroll
    for (int i = 0; i < NR; i++) {
        const int r = rg + 8 * i;
        s[i] = (live && r < D && pos > 0) ? S[(int64_t)r * V + c] : 0.0f;
    }
    // the first 128 inputs of the low-rank factors' rows are fetched ahead
    const int l8 = t & 7, r8 = t >> 3;
    uint4 fa[NR / 4][2], fg[2];
    float bias[NR / 4];
    const float rate = w.rate[h], beta = l_sigmoid(in[d.off_b() + h]);
#pragma unroll
    for (int i = 0; i < NR / 4; i++) bias[i] = r8 + 32 * i < D ? w.bias[h * D + r8 + 32 * i] : 0.0f;
#pragma unroll
    for (int i = 0; i < NR / 4; i++)
#pragma unroll
        for (int e = 0; e < 2; e++) {
            const int r = r8 + 32 * i, kk = 8 * l8 + 64 * e;
            fa[i][e] = make_uint4(0, 0, 0, 0);
            if (r < D && kk < w.lda2) fa[i][e] = *(const uint4 *)(w.a2 + ((int64_t)h * D + r) * w.lda2 + kk);
        }
#pragma unroll
    for (int e = 0; e < 2; e++) {
        const int kk = 8 * l8 + 64 * e;
        fg[e] = make_uint4(0, 0, 0, 0);
        if (c0 + r8 < V && kk < w.ldg2) fg[e] = *(const uint4 *)(w.g2 + ((int64_t)h * V + c0 + r8) * w.ldg2 + kk);
    }
    // short convolutions; the token's own projections go into the ring (its slot is not read by this token)
    const int C = d.channels(), now = pos % d.taps;
    float *slot = ring + (int64_t)now * C;
#pragma unroll
    for (int ii = 0; ii < (16 * NR + L_DELTA_COLS + 255) / 256; ii++) {
        const int i = t + 256 * ii;
        if (i >= 2 * D + L_DELTA_COLS) break;
        const bool isv = i >= 2 * D, isk = !isv && i >= D;
        const int e = isv ? i - 2 * D : isk ? i - D : i;
        if (isv && c0 + e >= V) {
            s_v[e] = 0.0f;
            continue;
        }
        const int ch = isv ? 2 * GD + h * V + c0 + e : (isk ? GD : 0) + kvh * D + e;
        const float cur = in[ch], y = delta_conv(w.conv, ring, C, d.taps, cur, ch, pos, now);
        if (isv)
            s_v[e] = y;
        else if (isk)
            s_k[e] = y;
        else
            s_q[e] = y;
        if (isv || (sp == 0 && h % (d.H / d.G) == 0)) slot[ch] = cur;
    }
    for (int i = t; i < w.lda2; i += 256) s_fa[i] = i < d.ra ? in[d.off_a() + i] : 0.0f;
    for (int i = t; i < w.ldg2; i += 256) s_fg[i] = i < d.rg ? in[d.off_g() + i] : 0.0f;
    __syncthreads();
    // unit vectors (one wavefront each), then k . q
    if (wave < 2) {
        float *x = wave ? s_k : s_q;
        float ss = 0.0f;
        for (int e = lane; e < D; e += 64) ss = fmaf(x[e], x[e], ss);
        float r = 1.0f / sqrtf(l_wave_sum(ss) + 1e-6f);
        if (wave == 0) r *= 1.0f / sqrtf((float)D);
        for (int e = lane; e < D; e += 64) x[e] *= r;
    }
    // decays of all key channels, gates of this workgroup's columns
#pragma unroll
    for (int i = 0; i < NR / 4; i++) {
        const int r = r8 + 32 * i;
        if (r >= D) break;
        const uint16_t *row = w.a2 + ((int64_t)h * D + r) * w.lda2;
        float z = 0.0f;
#pragma unroll
        for (int e = 0; e < 2; e++)
            if (8 * l8 + 64 * e < w.lda2) z = delta_fma8(fa[i][e], s_fa + 8 * l8 + 64 * e, z);
        for (int kk = 8 * l8 + 128; kk < w.lda2; kk += 64) z = delta_fma8(*(const uint4 *)(row + kk), s_fa + kk, z);
        z = delta_sum8(z) + bias[i];
        if (l8 == 0) s_g[r] = expf(-rate * l_softplus(z));
    }
    if (c0 + r8 < V) {
        const uint16_t *row = w.g2 + ((int64_t)h * V + c0 + r8) * w.ldg2;
        float z = 0.0f;
#pragma unroll
        for (int e = 0; e < 2; e++)
            if (8 * l8 + 64 * e < w.ldg2) z = delta_fma8(fg[e], s_fg + 8 * l8 + 64 * e, z);
        for (int kk = 8 * l8 + 128; kk < w.ldg2; kk += 64) z = delta_fma8(*(const uint4 *)(row + kk), s_fg + kk, z);
        z = delta_sum8(z);
        if (l8 == 0) gate[h * V + c0 + r8] = l_sigmoid(z);
    }
    __syncthreads();
    if (wave == 0) {
        float kq = 0.0f;
        for (int e = lane; e < D; e += 64) kq = fmaf(s_k[e], s_q[e], kq);
        kq = l_wave_sum(kq);
        if (lane == 0) s_kq = kq;
    }
    float dk = 0.0f, dq = 0.0f;
#pragma unroll
    for (int i = 0; i < NR; i++) {
        const int r = rg + 8 * i;
        if (r < D) {
            s[i] *= s_g[r];
            dk = fmaf(s[i], s_k[r], dk);
            dq = fmaf(s[i], s_q[r], dq);
        }
    }
    s_red[0][rg][col] = dk;
    s_red[1][rg][col] = dq;
    __syncthreads();
    dk = dq = 0.0f;
#pragma unroll
    for (int i = 0; i < 8; i++) {
        dk += s_red[0][i][col];
        dq += s_red[1][i][col];
    }
    const float u = beta * (s_v[col] - dk), ov = fmaf(s_kq, u, dq);
#pragma unroll
    for (int i = 0; i < NR; i++) {
        const int r = rg + 8 * i;
        if (live && r < D) S[(int64_t)r * V + c] = fmaf(s_k[r], u, s[i]);
    }
    if (rg == 0) {  // (the low half of wavefront 0)
        float ss = live ? ov * ov : 0.0f;
#pragma unroll
        for (int m = 16; m >= 1; m >>= 1) ss += __shfl_xor(ss, m, WAVE);
        if (live) o[h * V + c] = ov;
        if (col == 0) ssq[h * n_split + sp] = ss;
    }
}

hipError_t k_delta_step(hipStream_t s, const DeltaShape &d, const DeltaWeights &w, const float *in, float *ring, float *state,
                        const DecodeCtl *ctl, float *o, float *ssq, float *gate) {
    const int ns = delta_splits(d.V), nr = d.D <= 64 ? 8 : d.D <= 128 ? 16 : 32;
    if (d.D > 256) return hipErrorInvalidValue;
    const size_t lds = (size_t)(3 * 8 * nr + w.lda2 + w.ldg2) * sizeof(float);
    if (lds > 60 * 1024) return hipErrorInvalidValue;
    const dim3 grid((unsigned)ns, (unsigned)d.H);
#define GO(N) hipLaunchKernelGGL((delta_step_kernel<N>), grid, dim3(256), lds, s, d, w, in, ring, state, ctl, o, ssq, gate, ns)
    if (nr == 8)
        GO(8);
    else if (nr == 16)
        GO(16);
    else
        GO(32);
#undef GO
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------------------
// many tokens: convolutions and unit vectors.  A wavefront takes one unit (a key head's q and k, or a value head, or the
// rest of the row) over PREP_T consecutive tokens.
// ---------------------------------------------------------------------------------------------------------------
#define CH_T 16  // tokens of a chunk of the recurrence
#define PREP_T 8

// CONV_AHEAD - 1 + PREP_T inputs of a channel (tokens m0 - CONV_AHEAD + 1 .. m0 + PREP_T - 1) are fetched together, then the
// convolution and silu of its PREP_T tokens; taps beyond CONV_AHEAD are added one by one
__device__ __forceinline__ float delta_raw_at(const float *raw, int64_t ldr, const float *ring, int C, int taps, int ch, int m, int pos0) {
    if (m >= 0) return raw[(int64_t)m * ldr + ch];
    const int p = pos0 + m;
    return p >= 0 ? ring[(int64_t)(p % taps) * C + ch] : 0.0f;
}
__device__ __forceinline__ void delta_conv_rows(const float *conv, const float *raw, int64_t ldr, const float *ring, int C, int taps, int ch,
                                                int m0, int M, int pos0, float (&y)[PREP_T]) {
    float x[CONV_AHEAD - 1 + PREP_T], w[CONV_AHEAD];
    const float *col = raw + ch;
    if (m0 >= CONV_AHEAD - 1) {
#pragma unroll
        for (int i = 0; i < CONV_AHEAD - 1 + PREP_T; i++) x[i] = col[(int64_t)min(m0 - CONV_AHEAD + 1 + i, M - 1) * ldr];
    } else {
#pragma unroll
        for (int i = 0; i < CONV_AHEAD - 1 + PREP_T; i++) {
            const int m = m0 - CONV_AHEAD + 1 + i;
            // (an input further back than the taps reach has left the ring: its weight is 0)
            x[i] = (m >= 0 || -m < taps) ? delta_raw_at(raw, ldr, ring, C, taps, ch, min(m, M - 1), pos0) : 0.0f;
        }
    }
#pragma unroll
    for (int j = 0; j < CONV_AHEAD; j++) w[j] = j < taps ? conv[(int64_t)(taps - 1 - j) * C + ch] : 0.0f;
#pragma unroll
    for (int i = 0; i < PREP_T; i++) {
        float v = 0.0f;
#pragma unroll
        for (int j = 0; j < CONV_AHEAD; j++) v = fmaf(w[j], x[i + CONV_AHEAD - 1 - j], v);
        y[i] = v;
    }
    for (int j = CONV_AHEAD; j < taps; j++) {
        const float wj = conv[(int64_t)(taps - 1 - j) * C + ch];
        for (int i = 0; i < PREP_T; i++)
            if (m0 + i < M) y[i] = fmaf(wj, delta_raw_at(raw, ldr, ring, C, taps, ch, m0 + i - j, pos0), y[i]);
    }
#pragma unroll
    for (int i = 0; i < PREP_T; i++) y[i] = l_silu(y[i]);
}

// NE: key channels per lane (D <= 64 NE)
template <int PREC, int NE>
__global__ __launch_bounds__(256) void delta_prepare_kernel(DeltaShape d, const float *conv, const float *raw, int64_t ldr,
                                                            const float *ring, int M, int pos0, float *qkv, float *kq, float *beta,
                                                            void *fa, int64_t lfa, void *fg, int64_t lfg) {
    const int lane = threadIdx.x & 63;
    const int unit = blockIdx.x * 4 + (threadIdx.x >> 6), n_units = d.G + d.H + 1;
    const int m0 = blockIdx.y * PREP_T, m1 = min(m0 + PREP_T, M);
    if (unit >= n_units) return;
    const int C = d.channels(), GD = d.G * d.D, taps = d.taps;
    if (unit == d.G + d.H) {  // beta and the low-rank factors
        for (int m = m0; m < m1; m++) {
            const float *r = raw + (int64_t)m * ldr;
            for (int h = lane; h < d.H; h += 64) beta[(int64_t)m * d.H + h] = l_sigmoid(r[d.off_b() + h]);
            for (int i = lane; i < lfa; i += 64) l_store_act<PREC>(fa, (int64_t)m * lfa + i, i < d.ra ? r[d.off_a() + i] : 0.0f);
            for (int i = lane; i < lfg; i += 64) l_store_act<PREC>(fg, (int64_t)m * lfg + i, i < d.rg ? r[d.off_g() + i] : 0.0f);
        }
        return;
    }
    if (unit >= d.G) {  // a value head
        const int ch0 = 2 * GD + (unit - d.G) * d.V;
        for (int e = lane; e < d.V; e += 64) {
            float y[PREP_T];
            delta_conv_rows(conv, raw, ldr, ring, C, taps, ch0 + e, m0, M, pos0, y);
#pragma unroll
            for (int i = 0; i < PREP_T; i++)  // (rows of v are zero from M to the end of the last chunk)
                qkv[(int64_t)(m0 + i) * C + ch0 + e] = m0 + i < M ? y[i] : 0.0f;
        }
        return;
    }
    // a key head's q and k
    float q[NE][PREP_T], k[NE][PREP_T];
#pragma unroll
    for (int i = 0; i < NE; i++) {
        const int e = lane + 64 * i, ch = unit * d.D + min(e, d.D - 1);
        delta_conv_rows(conv, raw, ldr, ring, C, taps, ch, m0, M, pos0, q[i]);
        delta_conv_rows(conv, raw, ldr, ring, C, taps, GD + ch, m0, M, pos0, k[i]);
        if (e >= d.D)
#pragma unroll
            for (int j = 0; j < PREP_T; j++) q[i][j] = k[i][j] = 0.0f;
    }
    const float qs = 1.0f / sqrtf((float)d.D);
#pragma unroll
    for (int j = 0; j < PREP_T; j++) {
        float qq = 0.0f, kk = 0.0f, qk = 0.0f;
#pragma unroll
        for (int i = 0; i < NE; i++) {
            qq = fmaf(q[i][j], q[i][j], qq);
            kk = fmaf(k[i][j], k[i][j], kk);
            qk = fmaf(q[i][j], k[i][j], qk);
        }
        const float rq = qs / sqrtf(l_wave_sum(qq) + 1e-6f), rk = 1.0f / sqrtf(l_wave_sum(kk) + 1e-6f);
        qk = l_wave_sum(qk);
        const int m = m0 + j;
        if (m >= M) break;
#pragma unroll
        for (int i = 0; i < NE; i++) {
            const int e = lane + 64 * i;
            if (e >= d.D) continue;
            qkv[(int64_t)m * C + unit * d.D + e] = q[i][j] * rq;
            qkv[(int64_t)m * C + GD + unit * d.D + e] = k[i][j] * rk;
        }
        if (lane == 0) kq[(int64_t)m * d.G + unit] = qk * rq * rk;
    }
}

hipError_t k_delta_prepare(hipStream_t s, const DeltaShape &d, const float *conv, const float *raw, int64_t ldr, const float *ring,
                           int M, int pos0, float *qkv, float *kq, float *beta, void *fa, int64_t lfa, void *fg, int64_t lfg,
                           int prec) {
    if (d.D > 256 || M < 1) return hipErrorInvalidValue;
    const dim3 grid((unsigned)((d.G + d.H + 1 + 3) / 4), (unsigned)((M + CH_T - 1) / CH_T * (CH_T / PREP_T)));
#define GO(N)                                                                                                                            \
    do {                                                                                                                                 \
        if (prec)                                                                                                                        \
            hipLaunchKernelGGL((delta_prepare_kernel<1, N>), grid, dim3(256), 0, s, d, conv, raw, ldr, ring, M, pos0, qkv, kq, beta, fa, \
                               lfa, fg, lfg);                                                                                            \
        else                                                                                                                             \
            hipLaunchKernelGGL((delta_prepare_kernel<0, N>), grid, dim3(256), 0, s, d, conv, raw, ldr, ring, M, pos0, qkv, kq, beta, fa, \
                               lfa, fg, lfg);                                                                                            \
    } while (0)
    switch ((d.D + 63) / 64) {
    case 1: GO(1); break;
    case 2: GO(2); break;
    case 3: GO(3); break;
    default: GO(4); break;
    }
#undef GO
    return hipGetLastError();
}

// the ring takes the last `taps` tokens' projected channels
__global__ __launch_bounds__(256) void delta_ring_kernel(const float *raw, int64_t ldr, float *ring, int C, int taps, int M, int pos0) {
    const int ch = blockIdx.x * 256 + threadIdx.x, m = M - 1 - (int)blockIdx.y;
    if (ch >= C || m < 0) return;
    ring[(int64_t)((pos0 + m) % taps) * C + ch] = raw[(int64_t)m * ldr + ch];
}
hipError_t k_delta_ring(hipStream_t s, const DeltaShape &d, const float *raw, int64_t ldr, float *ring, int M, int pos0) {
    const int C = d.channels();
    hipLaunchKernelGGL(delta_ring_kernel, dim3((unsigned)((C + 255) / 256), (unsigned)std::min(M, d.taps)), dim3(256), 0, s, raw, ldr,
                       ring, C, d.taps, M, pos0);
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------------------
// the recurrence, token by token: workgroup (16 value columns, head); a wavefront holds 4 columns, 16 lanes per column,
// E = 4 NE key channels per lane (4 consecutive ones of every 64)
// ---------------------------------------------------------------------------------------------------------------
#define SCAN_T 16  // tokens staged in LDS at a time

// sum over the 16 lanes of a row, in every lane
__device__ __forceinline__ float row16_sum(float v) {
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x128, 0xF, 0xF, true));  // row_ror:8
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x124, 0xF, 0xF, true));
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x122, 0xF, 0xF, true));
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x121, 0xF, 0xF, true));
    return v;
}

template <int NE>
__global__ __launch_bounds__(256) void delta_scan_kernel(DeltaShape d, const float *qkv, const float *kq, const float *beta,
                                                         const float *lg, float *state, int M, int pos0, float *o) {
    constexpr int DP = 64 * NE;
    __shared__ __align__(16) float s_q[SCAN_T][DP], s_k[SCAN_T][DP], s_g[SCAN_T][DP];
    __shared__ float s_v[SCAN_T][16], s_o[SCAN_T][16], s_b[SCAN_T], s_kq[SCAN_T];
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6;
    const int h = blockIdx.y, kvh = h / (d.H / d.G), c0 = blockIdx.x * 16;
    const int D = d.D, V = d.V, C = d.channels(), GD = d.G * D;
    const int wc = 4 * wave + (lane >> 4), dl = lane & 15, c = c0 + wc;
    const bool live = c < V;
    float *S = state + (int64_t)h * D * V;
    float s[NE][4];
#pragma unroll
    for (int i = 0; i < NE; i++)
#pragma unroll
        for (int j = 0; j < 4; j++) {
            const int r = 64 * i + 4 * dl + j;
            s[i][j] = (live && r < D && pos0 > 0) ? S[(int64_t)r * V + c] : 0.0f;
        }
    for (int m0 = 0; m0 < M; m0 += SCAN_T) {
        const int n = min(SCAN_T, M - m0);
        __syncthreads();
        for (int i = t; i < SCAN_T * DP; i += 256) {
            const int tt = i / DP, e = i - tt * DP;
            float q = 0.0f, k = 0.0f, g = 1.0f;
            if (tt < n && e < D) {
                const float *row = qkv + (int64_t)(m0 + tt) * C + kvh * D + e;
                q = row[0];
                k = row[GD];
                g = expf(lg[(int64_t)(m0 + tt) * d.H * D + h * D + e]);
            }
            s_q[tt][e] = q;
            s_k[tt][e] = k;
            s_g[tt][e] = g;
        }
        {
            const int tt = t >> 4, e = t & 15;
            s_v[tt][e] = (tt < n && c0 + e < V) ? qkv[(int64_t)(m0 + tt) * C + 2 * GD + h * V + c0 + e] : 0.0f;
            if (e == 0) {
                s_b[tt] = tt < n ? beta[(int64_t)(m0 + tt) * d.H + h] : 0.0f;
                s_kq[tt] = tt < n ? kq[(int64_t)(m0 + tt) * d.G + kvh] : 0.0f;
            }
        }
        __syncthreads();
        for (int tt = 0; tt < n; tt++) {
            float4 k[NE], q[NE];
            float dk = 0.0f, dq = 0.0f;
#pragma unroll
            for (int i = 0; i < NE; i++) {
                const float4 g = *(const float4 *)&s_g[tt][64 * i + 4 * dl];
                k[i] = *(const float4 *)&s_k[tt][64 * i + 4 * dl];
                q[i] = *(const float4 *)&s_q[tt][64 * i + 4 * dl];
                s[i][0] *= g.x;
                s[i][1] *= g.y;
                s[i][2] *= g.z;
                s[i][3] *= g.w;
                dk = fmaf(s[i][0], k[i].x, dk);
                dq = fmaf(s[i][0], q[i].x, dq);
                dk = fmaf(s[i][1], k[i].y, dk);
                dq = fmaf(s[i][1], q[i].y, dq);
                dk = fmaf(s[i][2], k[i].z, dk);
                dq = fmaf(s[i][2], q[i].z, dq);
                dk = fmaf(s[i][3], k[i].w, dk);
                dq = fmaf(s[i][3], q[i].w, dq);
            }
            dk = row16_sum(dk);
            dq = row16_sum(dq);
            const float u = s_b[tt] * (s_v[tt][wc] - dk);
#pragma unroll
            for (int i = 0; i < NE; i++) {
                s[i][0] = fmaf(k[i].x, u, s[i][0]);
                s[i][1] = fmaf(k[i].y, u, s[i][1]);
                s[i][2] = fmaf(k[i].z, u, s[i][2]);
                s[i][3] = fmaf(k[i].w, u, s[i][3]);
            }
            if (dl == 0) s_o[tt][wc] = fmaf(s_kq[tt], u, dq);
        }
        __syncthreads();
        {
            const int tt = t >> 4, e = t & 15;
            if (tt < n && c0 + e < V) o[(int64_t)(m0 + tt) * d.H * V + h * V + c0 + e] = s_o[tt][e];
        }
    }
#pragma unroll
    for (int i = 0; i < NE; i++)
#pragma unroll
        for (int j = 0; j < 4; j++) {
            const int r = 64 * i + 4 * dl + j;
            if (live && r < D) S[(int64_t)r * V + c] = s[i][j];
        }
}

hipError_t k_delta_scan(hipStream_t s, const DeltaShape &d, const float *qkv, const float *kq, const float *beta, const float *lg,
                        float *state, int M, int pos0, float *o) {
    if (d.D > 256 || M < 1) return hipErrorInvalidValue;
    const dim3 grid((unsigned)((d.V + 15) / 16), (unsigned)d.H);
#define GO(N) hipLaunchKernelGGL((delta_scan_kernel<N>), grid, dim3(256), 0, s, d, qkv, kq, beta, lg, state, M, pos0, o)
    switch ((d.D + 63) / 64) {
    case 1: GO(1); break;
    case 2: GO(2); break;
    case 3: GO(3); break;
    default: GO(4); break;
    }
#undef GO
    return hipGetLastError();
}

// ---------------------------------------------------------------------------------------------------------------
// the recurrence in chunks of 16 tokens, on the fp32 matrix cores.  With G_i the decays' logarithms summed over the tokens
// 0 .. i of a chunk and S0 the state before it, unrolling the recurrence gives
//   A_ij = sum_d k_i k_j exp(G_i - G_j)  (j < i),   B_ij = sum_d q_i k_j exp(G_i - G_j)  (j <= i)
//   U = T (V - (k exp(G)) S0),  T = (I + diag(beta) A)^-1 diag(beta)
//   O = (q exp(G)) S0 + B U,    S = diag(exp(G_15)) S0 + (k exp(G_15 - G))^T U
// All exponents are <= 0.  A, B, T and the scaled rows depend on no state: delta_chunk_kernel makes them for all chunks at once;
// delta_walk_kernel then walks the chunks, 16 value columns a workgroup, the key channels split over its four wavefronts.
//
// Operands are stored in the order the lanes hold them.  v_mfma_f32_16x16x4_f32: lane l has A[l % 16][l / 16], B[l / 16][l % 16]
// and, of the result, rows 4 (l / 16) + r in register r, column l % 16.  With the four steps over a tile of 16 contracted
// indexes taken as k = 4 (l / 16) + r, a result is the next product's B operand as it stands, and an A operand's four steps are
// one 16-byte word of lane l: (row l % 16; columns 4 (l / 16) .. + 3).
// ---------------------------------------------------------------------------------------------------------------
typedef float d_f32x4 __attribute__((ext_vector_type(4)));

// the record of one (chunk, head): NT tiles of 16 key channels (a multiple of 4); kt, qt, kh: [NT][64][4]; T, B: [64][4];
// exp(G_15): [16 NT]
__host__ __device__ static inline int delta_chunk_tiles(int D) { return (D + 63) / 64 * 4; }
__host__ __device__ static inline int64_t delta_chunk_floats(int NT) { return (int64_t)NT * 784 + 512; }

template <int NW>
__global__ __launch_bounds__(256) void delta_chunk_kernel(DeltaShape d, const float *qkv, const float *beta, const float *lg, int M,
                                                          float *rec) {
    constexpr int NT = 4 * NW, DP = 16 * NT;
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6;
    // s_g: the decays, then their logarithms' sums
    __shared__ __align__(16) float s_q[CH_T * DP], s_k[CH_T * DP], s_g[CH_T * DP];
    __shared__ float s_A[CH_T][CH_T + 1], s_B[CH_T][CH_T + 1], s_T[CH_T][CH_T + 1], s_b[CH_T];
    const int ch = blockIdx.x, h = blockIdx.y, kvh = h / (d.H / d.G), m0 = ch * CH_T, n = min(CH_T, M - m0);
    const int D = d.D, C = d.channels(), GD = d.G * D;
    // a thread has one column of 16 / (256 / columns) rows at a time: column e, rows r0, r0 + RS, ...
    constexpr int CB = DP < 256 ? DP : 256, RS = 256 / CB, NR = CH_T / RS;  // (DP: 64, 128, 192 or 256)
    const int e0 = t % CB, r0 = t / CB;
    float l[NR];
    if (r0 < RS) {
        float q[NR], k[NR];
#pragma unroll
        for (int i = 0; i < NR; i++) {
            const int tt = r0 + RS * i;
            q[i] = k[i] = l[i] = 0.0f;
            if (tt < n && e0 < D) {
                const float *row = qkv + (int64_t)(m0 + tt) * C + kvh * D + e0;
                q[i] = row[0];
                k[i] = row[GD];
                l[i] = lg[((int64_t)(m0 + tt) * d.H + h) * D + e0];
            }
        }
#pragma unroll
        for (int i = 0; i < NR; i++) {
            const int at = (r0 + RS * i) * DP + e0;
            s_q[at] = q[i];
            s_k[at] = k[i];
            s_g[at] = expf(l[i]);
        }
    }
    if (t < CH_T) s_b[t] = t < n ? beta[(int64_t)(m0 + t) * d.H + h] : 0.0f;
    __syncthreads();
    // A and B: a group of 16 lanes has row j of the pairs (j, i > j), each lane every 16th channel; r = k_j times the decays of
    // the tokens after j
    {
        const int j = 4 * wave + (lane >> 4), sl = lane & 15;
        float a[CH_T], b[CH_T];
#pragma unroll
        for (int i = 0; i < CH_T; i++) a[i] = b[i] = 0.0f;
        for (int e = sl; e < D; e += 16) {
            float r = s_k[j * DP + e];
#pragma unroll
            for (int i = 0; i < CH_T; i++) {
                if (i > j) r *= s_g[i * DP + e];
                const float u = i >= j ? r : 0.0f;
                a[i] = fmaf(s_k[i * DP + e], u, a[i]);
                b[i] = fmaf(s_q[i * DP + e], u, b[i]);
            }
        }
#pragma unroll
        for (int i = 0; i < CH_T; i++) {
            a[i] = row16_sum(a[i]);
            b[i] = row16_sum(b[i]);
            if (sl == i) {
                s_A[i][j] = i > j ? a[i] : 0.0f;
                s_B[i][j] = b[i];
            }
        }
    }
    __syncthreads();
    // T by forward substitution, a lane per column
    if (t < CH_T) {
        float x[CH_T];
#pragma unroll
        for (int i = 0; i < CH_T; i++) {
            float v = i == t ? 1.0f : 0.0f;
#pragma unroll
            for (int j = 0; j < i; j++) v = fmaf(-s_A[i][j], x[j], v);
            x[i] = s_b[i] * v;
            s_T[i][t] = x[i];
        }
    }
    // sums of the logarithms, in place of the decays (whose readers are done)
    if (r0 < RS)
#pragma unroll
        for (int i = 0; i < NR; i++) s_g[(r0 + RS * i) * DP + e0] = l[i];
    __syncthreads();
    for (int e = t; e < DP; e += 256) {
        float g = 0.0f;
#pragma unroll
        for (int i = 0; i < CH_T; i++) {
            g += s_g[i * DP + e];
            s_g[i * DP + e] = g;
        }
    }
    __syncthreads();
    float *out = rec + ((int64_t)ch * d.H + h) * delta_chunk_floats(NT);
    for (int idx = t; idx < NT * 64; idx += 256) {
        const int tile = idx >> 6, l = idx & 63, row = l & 15, q4 = 4 * (l >> 4);
        float4 kt, qt, kh;
        {
            const int o = row * DP + 16 * tile + q4;
            const float4 k = *(const float4 *)(s_k + o), q = *(const float4 *)(s_q + o), G = *(const float4 *)(s_g + o);
            const float4 x = make_float4(expf(G.x), expf(G.y), expf(G.z), expf(G.w));
            kt = make_float4(k.x * x.x, k.y * x.y, k.z * x.z, k.w * x.w);
            qt = make_float4(q.x * x.x, q.y * x.y, q.z * x.z, q.w * x.w);
        }
        {  // row: the channel, columns: tokens
            const int e = 16 * tile + row;
            const float Gc = s_g[15 * DP + e];
            kh = make_float4(s_k[q4 * DP + e] * expf(Gc - s_g[q4 * DP + e]), s_k[(q4 + 1) * DP + e] * expf(Gc - s_g[(q4 + 1) * DP + e]),
                             s_k[(q4 + 2) * DP + e] * expf(Gc - s_g[(q4 + 2) * DP + e]),
                             s_k[(q4 + 3) * DP + e] * expf(Gc - s_g[(q4 + 3) * DP + e]));
        }
        *(float4 *)(out + 4 * idx) = kt;
        *(float4 *)(out + 256 * NT + 4 * idx) = qt;
        *(float4 *)(out + 512 * NT + 4 * idx) = kh;
    }
    if (t < 128) {
        const float(*m)[CH_T + 1] = wave ? s_B : s_T;
        const int row = lane & 15, q4 = 4 * (lane >> 4);
        *(float4 *)(out + 768 * NT + 256 * wave + 4 * lane) = make_float4(m[row][q4], m[row][q4 + 1], m[row][q4 + 2], m[row][q4 + 3]);
    }
    for (int e = t; e < DP; e += 256) out[768 * NT + 512 + e] = e < D ? expf(s_g[15 * DP + e]) : 0.0f;
}

// one chunk's operands of a wavefront with NW tiles of key channels
template <int NW>
struct DeltaOps {
    d_f32x4 kt[NW], qt[NW], kh[NW], gc[NW], T;
    float B, v[4];
};

// (records, rows of v and rows of o exist for whole chunks: a sequence's last chunk is filled up with zero rows)
template <int NW>
__global__ __launch_bounds__(256) void delta_walk_kernel(DeltaShape d, const float *rec, const float *qkv, float *state, int M, int pos0,
                                                         float *o, unsigned n_cb, unsigned n_items, unsigned per) {
    __shared__ __align__(16) d_f32x4 s_w[2][4][64];
    __shared__ float s_o[2][4][4][64];
    constexpr int NT = 4 * NW;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), col = lane & 15, q4 = 4 * (lane >> 4);
    // the workgroups of a head read the same records: they are dealt to one of the 8 XCDs (workgroups go to them in turn)
    const unsigned item = (blockIdx.x & 7u) * per + (blockIdx.x >> 3);
    if (item >= n_items) return;
    const int h = (int)(item / n_cb), c = (int)(item % n_cb) * 16 + col, D = d.D, V = d.V, C = d.channels(), HV = d.H * V;
    const bool live = c < V;
    float *S = state + (int64_t)h * D * V;
    d_f32x4 s[NW];
#pragma unroll
    for (int i = 0; i < NW; i++)
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const int e = 16 * (wave * NW + i) + q4 + r;
            s[i][r] = (live && e < D && pos0 > 0) ? S[(int64_t)e * V + c] : 0.0f;
        }
    const int n_ch = (M + CH_T - 1) / CH_T;
    // wavefront-uniform bases and this lane's fixed offsets from them
    const float *rec_h = rec + (int64_t)h * delta_chunk_floats(NT) + 256 * (wave * NW);
    const int64_t rec_step = (int64_t)d.H * delta_chunk_floats(NT);
    const float *v_h = qkv + 2 * d.G * D + h * V;
    float *o_h = o + (int64_t)wave * HV + h * V;
    const unsigned l4 = 4u * lane, ov = (unsigned)(q4 * HV + c);
    unsigned vv[4];
#pragma unroll
    for (int r = 0; r < 4; r++) vv[r] = (unsigned)((q4 + r) * C + (live ? c : 0));
    auto fetch = [&](DeltaOps<NW> &x, int ch) {
        const float *p = rec_h + ch * rec_step;
#pragma unroll
        for (int i = 0; i < NW; i++) {
            x.kt[i] = *(const d_f32x4 *)(p + 256 * i + l4);
            x.qt[i] = *(const d_f32x4 *)(p + 256 * (NT + i) + l4);
            x.kh[i] = *(const d_f32x4 *)(p + 256 * (2 * NT + i) + l4);
        }
        p -= 256 * (wave * NW);
#pragma unroll
        for (int i = 0; i < NW; i++) x.gc[i] = *(const d_f32x4 *)(p + 768 * NT + 512 + 16 * (wave * NW + i) + q4);
        x.T = *(const d_f32x4 *)(p + 768 * NT + l4);
        x.B = (p + wave)[768 * NT + 256 + l4];
        const float *v = v_h + (int64_t)ch * CH_T * C;
#pragma unroll
        for (int r = 0; r < 4; r++) x.v[r] = v[vv[r]];
    };
    // the output row 4 (lane / 16) + wave of a chunk, from the four wavefronts' parts
    auto put = [&](int ch) {
        const int b = ch & 1;
        const float y = s_o[b][wave][0][lane] + s_o[b][wave][1][lane] + s_o[b][wave][2][lane] + s_o[b][wave][3][lane];
        if (live) (o_h + (int64_t)ch * CH_T * HV)[ov] = y;
    };
    auto walk = [&](DeltaOps<NW> &x, int ch) {
        const int b = ch & 1;
        d_f32x4 w = {0.f, 0.f, 0.f, 0.f}, y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < NW; i++)
#pragma unroll
            for (int r = 0; r < 4; r++) w = __builtin_amdgcn_mfma_f32_16x16x4f32(x.kt[i][r], s[i][r], w, 0, 0, 0);
        s_w[b][wave][lane] = w;
#pragma unroll
        for (int i = 0; i < NW; i++)
#pragma unroll
            for (int r = 0; r < 4; r++) y = __builtin_amdgcn_mfma_f32_16x16x4f32(x.qt[i][r], s[i][r], y, 0, 0, 0);
        // LDS writes done, then the barrier (which also says that the parts of the previous chunk's output are all there);
        // the operands under way from memory are not waited for
        asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
        w = s_w[b][0][lane] + s_w[b][1][lane] + s_w[b][2][lane] + s_w[b][3][lane];
        d_f32x4 u = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int r = 0; r < 4; r++) u = __builtin_amdgcn_mfma_f32_16x16x4f32(x.T[r], x.v[r] - w[r], u, 0, 0, 0);
#pragma unroll
        for (int i = 0; i < NW; i++) {
            s[i] *= x.gc[i];
#pragma unroll
            for (int r = 0; r < 4; r++) s[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.kh[i][r], u[r], s[i], 0, 0, 0);
        }
        // B U: this wavefront's quarter of the contracted tokens
        const float uw = wave == 0 ? u[0] : wave == 1 ? u[1] : wave == 2 ? u[2] : u[3];
        y = __builtin_amdgcn_mfma_f32_16x16x4f32(x.B, uw, y, 0, 0, 0);
        if (ch) put(ch - 1);
#pragma unroll
        for (int r = 0; r < 4; r++) s_o[b][r][wave][lane] = y[r];
    };
    // the operands of three chunks are held or under way
    DeltaOps<NW> x0, x1, x2;
    fetch(x0, 0);
    fetch(x1, min(1, n_ch - 1));
    fetch(x2, min(2, n_ch - 1));
    for (int ch = 0; ch < n_ch; ch += 3) {  // (n_ch is the same for every wavefront: so is every barrier)
        walk(x0, ch);
        fetch(x0, min(ch + 3, n_ch - 1));
        if (ch + 1 >= n_ch) break;
        walk(x1, ch + 1);
        fetch(x1, min(ch + 4, n_ch - 1));
        if (ch + 2 >= n_ch) break;
        walk(x2, ch + 2);
        fetch(x2, min(ch + 5, n_ch - 1));
    }
    __syncthreads();
    put(n_ch - 1);
#pragma unroll
    for (int i = 0; i < NW; i++)
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const int e = 16 * (wave * NW + i) + q4 + r;
            if (live && e < D) S[(int64_t)e * V + c] = s[i][r];
        }
}

int64_t delta_walk_floats(const DeltaShape &d, int M) {
    return (int64_t)((M + CH_T - 1) / CH_T) * d.H * delta_chunk_floats(delta_chunk_tiles(d.D));
}
hipError_t k_delta_walk(hipStream_t s, const DeltaShape &d, const float *qkv, const float *beta, const float *lg, float *state, int M,
                        int pos0, float *rec, float *o) {
    if (d.D > 256 || M < 1) return hipErrorInvalidValue;
    const dim3 g1((unsigned)((M + CH_T - 1) / CH_T), (unsigned)d.H);
    const unsigned n_cb = (unsigned)((d.V + 15) / 16), n_items = n_cb * (unsigned)d.H, per = (n_items + 7) / 8;
#define GO(N)                                                                                                                      \
    do {                                                                                                                           \
        hipLaunchKernelGGL((delta_chunk_kernel<N>), g1, dim3(256), 0, s, d, qkv, beta, lg, M, rec);                                \
        hipLaunchKernelGGL((delta_walk_kernel<N>), dim3(8 * per), dim3(256), 0, s, d, rec, qkv, state, M, pos0, o, n_cb, n_items, per); \
    } while (0)
    switch (delta_chunk_tiles(d.D) / 4) {
    case 1: GO(1); break;
    case 2: GO(2); break;
    case 3: GO(3); break;
    default: GO(4); break;
    }
#undef GO
    return hipGetLastError();
}

// one wavefront per (token, head)
template <int PREC>
__global__ __launch_bounds__(256) void head_norm_rows_kernel(const float *o, const float *gate, const float *normw, int M, int H, int V,
                                                             float eps, void *outa, int64_t lda) {
    const int lane = threadIdx.x & 63;
    const int64_t unit = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (unit >= (int64_t)M * H) return;
    const int m = (int)(unit / H), h = (int)(unit - (int64_t)m * H);
    const float *x = o + (int64_t)m * H * V + h * V, *g = gate + (int64_t)m * H * V + h * V;
    float ss = 0.0f;
    for (int j = lane; j < V; j += 64) ss = fmaf(x[j], x[j], ss);
    const float r = 1.0f / sqrtf(l_wave_sum(ss) / (float)V + eps);
    for (int j = lane; j < V; j += 64) l_store_act<PREC>(outa, m * lda + h * V + j, x[j] * r * normw[j] * g[j]);
    if (h == H - 1)
        for (int64_t j = (int64_t)H * V + lane; j < lda; j += 64) l_store_act<PREC>(outa, m * lda + j, 0.0f);
}
hipError_t k_head_norm_rows(hipStream_t s, const float *o, const float *gate, const float *normw, int M, int H, int V, float eps,
                            void *outa, int64_t lda, int prec) {
    const dim3 grid((unsigned)(((int64_t)M * H + 3) / 4));
    if (prec)
        hipLaunchKernelGGL((head_norm_rows_kernel<1>), grid, dim3(256), 0, s, o, gate, normw, M, H, V, eps, outa, lda);
    else
        hipLaunchKernelGGL((head_norm_rows_kernel<0>), grid, dim3(256), 0, s, o, gate, normw, M, H, V, eps, outa, lda);
    return hipGetLastError();
}
