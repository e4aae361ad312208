// The many-token products of k_gemm.hip from tile images of the weights (pf_tile.h), bf16 activations: fused epilogues and the
// grouped form for mixtures of experts.
#include "layered_gemm.h"
#include "pf_tile.h"

// One thread copies a 16-byte chunk of an image: n_mats matrices of `rows` rows, each padded to whole tiles of 256 rows.
__global__ __launch_bounds__(256) void tile_image_kernel(const uint16_t *w, int ld, int64_t rows, int64_t n_chunks, uint16_t *dst) {
    const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (idx >= n_chunks) return;
    const int64_t nk = ld >> 6, nt_per = (rows + 255) / 256;
    const int within = (int)(idx & 2047), r = within >> 3, c = (within & 7) ^ pf_swz(r);
    const int64_t tile = idx >> 11, kt = tile % nk, ntm = tile / nk, nt = ntm % nt_per, mat = ntm / nt_per;
    const int64_t row = nt * 256 + r;
    uint4 v = make_uint4(0, 0, 0, 0);
    if (row < rows) v = *(const uint4 *)(w + (mat * rows + row) * ld + kt * 64 + 8 * c);
    ((uint4 *)dst)[idx] = v;
}
int64_t k_tile_image_elems(int64_t rows, int ld) { return (rows + 255) / 256 * 256 * ld; }
hipError_t k_tile_image(hipStream_t s, const uint16_t *w, int ld, int64_t rows, int64_t n_mats, uint16_t *dst) {
    if (ld % 64 != 0 || rows < 1) return hipErrorInvalidValue;
    const int64_t n = n_mats * k_tile_image_elems(rows, ld) / 8;
    if ((n + 255) / 256 > 0x7FFFFFFF) return hipErrorInvalidValue;
    hipLaunchKernelGGL(tile_image_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, s, w, ld, rows, n, dst);
    return hipGetLastError();
}

// 256 rows of the matrix (row group nt of w) x the positions m0 .. of a block of mcount, which starts at row mb
template <int EPI, int JT>
__device__ __forceinline__ void tiles_item(const GemmArgs &a, const uint16_t *w, unsigned nt, int64_t mb, int m0, int mcount, uint4 *s_all) {
    const int64_t n0 = (int64_t)nt * 256;
    pf_tile_product<JT>(
        w + (int64_t)nt * (a.ld >> 6) * 16384, (const uint16_t *)a.x, a.ld, s_all,
        [&](int r) {
            const int64_t row = mb + min(m0 + r, mcount - 1);  // (rows past the end repeat the last one; not stored)
            return a.gather ? (int64_t)a.gather[row] : row;
        },
        [&](f32x16(&acc)[2][JT], int wn, int wm, int lane) {
#pragma unroll
            for (int j = 0; j < JT; j++) {
                const int m = m0 + 32 * JT * wm + 32 * j + (lane & 31);
                if (m >= mcount) continue;
#pragma unroll
                for (int i = 0; i < 2; i++)
#pragma unroll
                    for (int rq = 0; rq < 4; rq++)
                        gemm_store4<0, EPI>(a, mb + m, n0 + 64 * wn + 32 * i + 8 * rq + 4 * (lane >> 5), acc[i][j][4 * rq],
                                            acc[i][j][4 * rq + 1], acc[i][j][4 * rq + 2], acc[i][j][4 * rq + 3]);
            }
        });
}

// Items (row group of 256, block of 64 JT positions) are dealt to the 8 XCDs as contiguous runs: positions fastest in a single
// product, so that workgroups on one weight tile share an L2; row groups fastest in a grouped one, where a block of positions
// is used with one expert's matrix only.
template <int EPI, int JT, bool GROUPED>
__global__ __launch_bounds__(512) void tiles_kernel(GemmArgs a, unsigned n_nt, unsigned n_mt) {
    extern __shared__ uint4 s_all[];
    const unsigned n_items = GROUPED ? (unsigned)a.n_tiles[0] * n_nt : n_nt * n_mt;
    const unsigned per = (n_items + 7) / 8, k = blockIdx.x >> 3, item = (blockIdx.x & 7u) * per + k;
    if (k >= per || item >= n_items) return;
    unsigned nt;
    int64_t mb = 0;
    int m0 = 0, mcount = a.M;
    const uint16_t *w = a.w;
    if (GROUPED) {
        const GemmTile g = a.tiles[item / n_nt];
        nt = item % n_nt;
        w += g.expert * a.expert_stride;
        mb = g.row0;
        mcount = g.n;
    } else {
        nt = item / n_mt;
        m0 = (int)(item % n_mt) * 64 * JT;
    }
    // (a block of a grouped product that has at most 128 rows takes half the positions)
    if (GROUPED && JT == 4 && mcount <= 128)
        tiles_item<EPI, 2>(a, w, nt, mb, m0, mcount, s_all);
    else
        tiles_item<EPI, JT>(a, w, nt, mb, m0, mcount, s_all);
}

#define TILES_MAX_DEVICES 64

template <int EPI, int JT, bool GROUPED>
static hipError_t tiles_launch(hipStream_t s, const GemmArgs &a, unsigned n_nt, unsigned n_mt) {
    constexpr int lds = 2 * (32768 + 64 * JT * 128);
    int dev = 0;
    hipError_t e = hipGetDevice(&dev);
    if (e != hipSuccess) return e;
    if (dev < 0 || dev >= TILES_MAX_DEVICES) return hipErrorInvalidDevice;
    static bool attr_set[TILES_MAX_DEVICES] = {};
    if (!attr_set[dev]) {
        e = hipFuncSetAttribute((const void *)tiles_kernel<EPI, JT, GROUPED>, hipFuncAttributeMaxDynamicSharedMemorySize, lds);
        if (e != hipSuccess) return e;
        attr_set[dev] = true;
    }
    const unsigned most = GROUPED ? (unsigned)a.max_tiles * n_nt : n_nt * n_mt;
    hipLaunchKernelGGL((tiles_kernel<EPI, JT, GROUPED>), dim3(8 * ((most + 7) / 8)), dim3(512), lds, s, a, n_nt, n_mt);
    return hipGetLastError();
}

// a.w: the image; otherwise as k_gemm with bf16 activations (ldx == ld)
hipError_t k_tiles(hipStream_t s, const GemmArgs &args, int epi) {
    GemmArgs a = args;
    if (!a.acols) a.acols = a.lda;
    if (!a.w || !a.x || a.n_rows < 1 || a.M < 1 || a.ld % 64 != 0 || a.ldx != a.ld || a.lda % 64 != 0 || a.acols % 64 != 0 ||
        a.acols > a.lda)
        return hipErrorInvalidValue;
    const unsigned n_nt = (unsigned)((a.n_rows + 255) / 256);
    const bool covered = a.outa && a.acols >= a.n_rows && a.acols <= 256 * (int64_t)n_nt;
    const bool pairs = a.outa && a.n_rows % 2 == 0 && 2 * a.acols >= a.n_rows && 2 * a.acols <= 256 * (int64_t)n_nt;
    if (a.tiles) {
        if (epi == GE_UP && covered) return tiles_launch<GE_UP, 4, true>(s, a, n_nt, 0);
        if (epi == GE_GLU && pairs) return tiles_launch<GE_GLU, 4, true>(s, a, n_nt, 0);
        if (epi == GE_STORE && a.outf && a.ldo >= a.n_rows) return tiles_launch<GE_STORE, 4, true>(s, a, n_nt, 0);
        return hipErrorInvalidValue;
    }
    if (!(epi == GE_ACT && covered) && !(epi == GE_GLU && pairs)) return hipErrorInvalidValue;
    const unsigned n_mt4 = (unsigned)((a.M + 255) / 256), n_mt2 = (unsigned)((a.M + 127) / 128);
    if (epi == GE_GLU)
        return n_nt * n_mt4 >= 256 ? tiles_launch<GE_GLU, 4, false>(s, a, n_nt, n_mt4) : tiles_launch<GE_GLU, 2, false>(s, a, n_nt, n_mt2);
    if (n_nt * n_mt4 >= 256) return tiles_launch<GE_ACT, 4, false>(s, a, n_nt, n_mt4);
    return tiles_launch<GE_ACT, 2, false>(s, a, n_nt, n_mt2);
}
