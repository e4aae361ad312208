// The bf16 tile product of the prompt pass (gfx950 matrix cores), shared by the kernels that run it.
#pragma once

#include "dev_common.h"

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x2 __attribute__((ext_vector_type(2)));
typedef float f32x16 __attribute__((ext_vector_type(16)));

__device__ __forceinline__ uint32_t pack_bf16(float a, float b) {
    bf16x2 v;
    v.x = (__bf16)a;
    v.y = (__bf16)b;
    return __builtin_bit_cast(uint32_t, v);
}
__device__ __forceinline__ bf16x8 as_bf16x8(uint4 v) { return __builtin_bit_cast(bf16x8, v); }

// Placement of the 16-byte chunks of a 128-byte tile row in LDS.  The LDS has 64 banks of 4 bytes and serves
// 16-byte accesses 16 lanes at a time; lanes read one chunk index of 16 consecutive rows, which the
// exclusive-or with (r >> 1) % 8 sends to the 16 different 16-byte slots of the 256-byte bank row (the row's
// parity picks the half).  With r % 8 instead, rows r and r + 8 collide: half the LDS cycles were conflicts.
__host__ __device__ __forceinline__ int pf_swz(int r) { return (r >> 1) & 7; }

#define PF_AS1 __attribute__((address_space(1)))
#define PF_AS3 __attribute__((address_space(3)))

// Product of bf16 tiles prepared beforehand (32 KB images of 256 weight rows x 64 inputs, 16-byte chunk c of row r at chunk
// index 8 r + (c ^ pf_swz(r))): no arithmetic on the operands.  A workgroup's tile is 256 weight rows
// x 64 JT positions (JT = 4: 256 positions, 64 KB fetched per 64 inputs, half the bytes per product of a 128 x 128 tile; JT = 2: 128 positions, for matrices with too few rows to give
// every CU a 256 x 256 tile), worked on by 8 wavefronts, 4 row groups x 2 position groups, each 64 rows x
// 32 JT positions.  Both operand tiles of a K step travel from global memory
// straight into LDS (16 bytes per lane and load, a wavefront's load filling 1 KB in lane order): the weight
// tile is a linear copy of its 32 KB image, the position tile gets the c ^ pf_swz(r) placement by the choice
// of the address each lane reads.  Two LDS stages: the loads of step kt + 1 are in flight during the products
// of step kt, one barrier per step.
typedef uint32_t pf_u32x4 __attribute__((ext_vector_type(4)));

// wtiles: the row group's tiles, K / 64 of them in a row; act: bf16 rows of K elements; s_all: two stages of LDS.  row(r) is the
// activation row of the tile's position r; epi(acc, wn, wm, lane) takes the results: a lane holds position
// 32 JT wm + 32 j + lane % 32 and, in register r of tile i, weight row 64 wn + 32 i + 8 (r / 4) + 4 (lane / 32) + r % 4.
template <int JT, class Row, class Epi>
__device__ __forceinline__ void pf_tile_product(const uint16_t *wtiles, const uint16_t *act, int64_t K, uint4 *s_all, Row row, Epi epi) {
    constexpr int MT = 64 * JT;                   // positions per workgroup
    constexpr int STAGE = 32768 + MT * 128;       // bytes: weight tile, then position tile
    const int t = threadIdx.x, lane = t & 63, wave = __builtin_amdgcn_readfirstlane(t >> 6), wn = wave & 3, wm = wave >> 2;
    const int64_t nk = K >> 6;

    // weights: this wavefront copies bytes [4096 wave, +4096) of every tile, 1 KB per load
    const unsigned char *gw = (const unsigned char *)wtiles + wave * 4096 + lane * 16;
    // positions: load i of this wavefront fills chunks 64 (JT wave + i) + lane: row 8 (JT wave + i) + lane / 8,
    // placed chunk lane % 8 = the data chunk (lane % 8) ^ pf_swz(row)
    const unsigned char *gx[JT];
#pragma unroll
    for (int i = 0; i < JT; i++) {
        const int r = 8 * (JT * wave + i) + (lane >> 3);
        gx[i] = (const unsigned char *)(act + row(r) * K + 8 * ((lane & 7) ^ pf_swz(r)));
    }
    // LDS byte offsets of this lane's operands inside a stage: slice kk holds chunk 2 kk + lane / 32 of its rows
    unsigned aw[2][4], ax[JT][4];
#pragma unroll
    for (int kk = 0; kk < 4; kk++) {
        const int c = 2 * kk + (lane >> 5);
#pragma unroll
        for (int i = 0; i < 2; i++) {
            const int ra = 64 * wn + 32 * i + (lane & 31);
            aw[i][kk] = 16u * (unsigned)(ra * 8 + (c ^ pf_swz(ra)));
        }
#pragma unroll
        for (int j = 0; j < JT; j++) {
            const int rb = 32 * JT * wm + 32 * j + (lane & 31);
            ax[j][kk] = 32768u + 16u * (unsigned)(rb * 8 + (c ^ pf_swz(rb)));
        }
    }
    const unsigned lds0 = (unsigned)(size_t)s_all;

    f32x16 acc[2][JT];
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int j = 0; j < JT; j++)
#pragma unroll
            for (int r = 0; r < 16; r++) acc[i][j][r] = 0.0f;

    auto issue = [&](int stage) {
        unsigned char *lw = (unsigned char *)s_all + stage * STAGE + wave * 4096;
        unsigned char *lx = (unsigned char *)s_all + stage * STAGE + 32768 + wave * (1024 * JT);
        __builtin_amdgcn_global_load_lds((const PF_AS1 void *)gw, (PF_AS3 void *)lw, 16, 0, 0);
        __builtin_amdgcn_global_load_lds((const PF_AS1 void *)gw, (PF_AS3 void *)lw, 16, 1024, 0);
        __builtin_amdgcn_global_load_lds((const PF_AS1 void *)gw, (PF_AS3 void *)lw, 16, 2048, 0);
        __builtin_amdgcn_global_load_lds((const PF_AS1 void *)gw, (PF_AS3 void *)lw, 16, 3072, 0);
#pragma unroll
        for (int i = 0; i < JT; i++) {
            __builtin_amdgcn_global_load_lds((const PF_AS1 void *)gx[i], (PF_AS3 void *)(lx + 1024 * i), 16, 0, 0);
            gx[i] += 128;
        }
        gw += 32768;
    };

    // The operands of a 16-wide slice (2 weight groups, JT position groups) are read from LDS one slice ahead
    // of the products that use them, into two register sets used in turn, so that a wavefront's LDS latency
    // lies under its own products.  Reads and waits are asm: the compiler then does not make them wait for the
    // copies in flight into the other stage.  Between a PF_READ and the PF_WAIT that retires it the registers
    // of the set hold nothing yet: the set only appears as an operand of those two statements and of the
    // products after the wait (LDS reads complete in order, so lgkmcnt(2 + JT) retires all but the newest set;
    // the build's asm check walks the generated code for any other touch of such a register).
    pf_u32x4 F0[2 + JT], F1[2 + JT];
#define PF_READ(F, KK)                                                                                            \
    do {                                                                                                          \
        if constexpr (JT == 2)                                                                                    \
            asm volatile("ds_read_b128 %0, %4\n\tds_read_b128 %1, %5\n\tds_read_b128 %2, %6\n\tds_read_b128 %3, %7"  \
                         : "=&v"(F[0]), "=&v"(F[1]), "=&v"(F[2]), "=&v"(F[3])                                     \
                         : "v"(sb + aw[0][KK]), "v"(sb + aw[1][KK]), "v"(sb + ax[0][KK]), "v"(sb + ax[1][KK])     \
                         : "memory");                                                                             \
        else                                                                                                      \
            asm volatile("ds_read_b128 %0, %6\n\tds_read_b128 %1, %7\n\tds_read_b128 %2, %8\n\tds_read_b128 %3, %9"  \
                         "\n\tds_read_b128 %4, %10\n\tds_read_b128 %5, %11"                                       \
                         : "=&v"(F[0]), "=&v"(F[1]), "=&v"(F[2]), "=&v"(F[3]), "=&v"(F[4]), "=&v"(F[5])           \
                         : "v"(sb + aw[0][KK]), "v"(sb + aw[1][KK]), "v"(sb + ax[0][KK]), "v"(sb + ax[1][KK]),    \
                           "v"(sb + ax[JT - 2][KK]), "v"(sb + ax[JT - 1][KK])                                     \
                         : "memory");                                                                             \
    } while (0)
    // LAST: nothing newer is in flight
#define PF_WAIT(F, LAST)                                                                                          \
    do {                                                                                                          \
        if constexpr (JT == 2) {                                                                                  \
            if (LAST)                                                                                             \
                asm volatile("s_waitcnt lgkmcnt(0)" : "+v"(F[0]), "+v"(F[1]), "+v"(F[2]), "+v"(F[3])::"memory");  \
            else                                                                                                  \
                asm volatile("s_waitcnt lgkmcnt(4)" : "+v"(F[0]), "+v"(F[1]), "+v"(F[2]), "+v"(F[3])::"memory");  \
        } else {                                                                                                  \
            if (LAST)                                                                                             \
                asm volatile("s_waitcnt lgkmcnt(0)"                                                               \
                             : "+v"(F[0]), "+v"(F[1]), "+v"(F[2]), "+v"(F[3]), "+v"(F[JT]), "+v"(F[JT + 1])::"memory"); \
            else                                                                                                  \
                asm volatile("s_waitcnt lgkmcnt(6)"                                                               \
                             : "+v"(F[0]), "+v"(F[1]), "+v"(F[2]), "+v"(F[3]), "+v"(F[JT]), "+v"(F[JT + 1])::"memory"); \
        }                                                                                                         \
    } while (0)
#define PF_PRODUCTS(F)                                                                                            \
    do {                                                                                                          \
        const bf16x8 W0 = __builtin_bit_cast(bf16x8, F[0]), W1 = __builtin_bit_cast(bf16x8, F[1]);                \
        _Pragma("unroll") for (int j = 0; j < JT; j++) {                                                          \
            const bf16x8 P = __builtin_bit_cast(bf16x8, F[2 + j]);                                                \
            acc[0][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(W0, P, acc[0][j], 0, 0, 0);                       \
            acc[1][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(W1, P, acc[1][j], 0, 0, 0);                       \
        }                                                                                                         \
    } while (0)

    issue(0);
    for (int64_t kt = 0; kt < nk; kt++) {
        const int stage = (int)(kt & 1);
        // this wavefront's loads of the stage have landed; the barrier says the same of the others' and that
        // everyone is done reading the other stage (its last PF_WAIT retired every read), which the next loads
        // then overwrite
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __builtin_amdgcn_s_barrier();
        if (kt + 1 < nk) issue(stage ^ 1);
        const unsigned sb = lds0 + (unsigned)(stage * STAGE);
        PF_READ(F0, 0);
        PF_READ(F1, 1);
        PF_WAIT(F0, false);
        PF_PRODUCTS(F0);
        PF_READ(F0, 2);
        PF_WAIT(F1, false);
        PF_PRODUCTS(F1);
        PF_READ(F1, 3);
        PF_WAIT(F0, false);
        PF_PRODUCTS(F0);
        PF_WAIT(F1, true);
        PF_PRODUCTS(F1);
    }
#undef PF_PRODUCTS
#undef PF_WAIT
#undef PF_READ
    epi(acc, wn, wm, lane);
}

