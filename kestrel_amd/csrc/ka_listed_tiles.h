// A tile of a matrix product whose activation rows are named by a list (gathered rows), with both operands staged through
// LDS: 128 list rows by 256 weight rows a workgroup of 256 threads, bf16 operands, fp32 sums on v_mfma_f32_32x32x16_bf16, any K
// that is a multiple of 16.
//
// The threads fetch a slab of 64 channels of the tile's 128 list rows and 256 weight rows by whole 128-byte lines (eight
// lanes a row), once for all four waves, into registers while the slab before is multiplied, then into the other of two
// LDS buffers; a wave reads its operands from there, 16 bytes a lane (rows 144 bytes apart, so that the 16 lanes of a pass
// fall on all banks). One barrier a slab, which waits for LDS alone. A last slab that ends before its 64 channels is filled
// with zeros (TAIL).
//
// A wave owns 64 weight rows (two blocks of 32) and all 128 list rows (four blocks of 32): acc[wb][rb]. With swap[wb] false
// the weights are the row operand of the product: a lane holds, of list row 32 rb + lane % 32, the weight rows
// 32 wb + (i / 4) 8 + (lane / 32) 4 + i % 4 in register i. With swap[wb] true the list rows are: a lane holds, of weight row
// 32 wb + lane % 32, the list rows 32 rb + (i / 4) 8 + (lane / 32) 4 + i % 4.
#pragma once

#include "ka_common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 kl_bf16x8;
typedef __attribute__((ext_vector_type(4))) __bf16 kl_bf16x4;
typedef __attribute__((ext_vector_type(16))) float kl_floatx16;

constexpr int KL_ROWS = 128;                                   // list rows a workgroup (and a tile of a list)
constexpr int KL_COLS = 256;                                   // weight rows a workgroup
constexpr int KL_SLAB = 64;
constexpr int KL_PITCH = KL_SLAB + 8;                          // bf16 numbers from one LDS row to the next
constexpr int KL_STAGE = (KL_ROWS + KL_COLS) * KL_PITCH;       // numbers of one buffer: the list rows, then the weight rows
constexpr int KL_LDS_BYTES = 2 * KL_STAGE * (int)sizeof(bf16_t);

// list_row(r), weight_row(r): the first channel of the tile's list row r (0 .. 127) and weight row r (0 .. 255), valid for
// loads whatever r is. computes: whether this wave has weight rows to multiply (it stages all the same).
template <bool TAIL, bool MAY_SWAP, typename ListRow, typename WeightRow>
__device__ __forceinline__ void kl_tile_product(bf16_t* lds, int K, bool computes, const bool (&swap)[2], ListRow list_row,
                                                WeightRow weight_row, kl_floatx16 (&acc)[2][4]) {
    const int tid = threadIdx.x, wave = tid / KA_WAVE, lane = tid % KA_WAVE;
    const int col = lane % 32, half = lane / 32;
    // what this thread fetches of every slab: piece tid % 8 (16 bytes) of the rows tid / 8 + 32 i: four list rows, eight
    // weight rows
    const int piece = tid % 8, row0 = tid / 8;
    const bf16_t* src[12];
    int dst[12];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        src[i] = list_row(row0 + 32 * i);
        dst[i] = (row0 + 32 * i) * KL_PITCH + piece * 8;
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) {
        src[4 + i] = weight_row(row0 + 32 * i);
        dst[4 + i] = (KL_ROWS + row0 + 32 * i) * KL_PITCH + piece * 8;
    }
#pragma unroll
    for (int wb = 0; wb < 2; ++wb)
#pragma unroll
        for (int rb = 0; rb < 4; ++rb)
#pragma unroll
            for (int i = 0; i < 16; ++i) acc[wb][rb][i] = 0.f;
    kl_bf16x8 st[12];
    auto fetch = [&](int kk) {
        const int at = kk + piece * 8;
        const bool in = !TAIL || at < K;           // (a piece behind the last channel: any address of the row, zeroed below)
#pragma unroll
        for (int i = 0; i < 12; ++i) st[i] = *reinterpret_cast<const kl_bf16x8*>(src[i] + (in ? at : 0));
    };
    auto stage = [&](int buf, int kk) {
        if constexpr (TAIL) {
            // (here and not where they are asked for, which would wait for them ahead of the products)
            if (kk + KL_SLAB > K) {
                const bool in = kk + piece * 8 < K;
#pragma unroll
                for (int i = 0; i < 12; ++i)
#pragma unroll
                    for (int u = 0; u < 8; ++u) st[i][u] = in ? st[i][u] : (bf16_t)0.f;
            }
        }
#pragma unroll
        for (int i = 0; i < 12; ++i) *reinterpret_cast<kl_bf16x8*>(lds + buf * KL_STAGE + dst[i]) = st[i];
    };
    auto lds_barrier = [&]() {
        __builtin_amdgcn_s_waitcnt(0xc07f);      // lgkmcnt(0), the other counters at their maximum
        asm volatile("" ::: "memory");
        __builtin_amdgcn_s_barrier();
        asm volatile("" ::: "memory");
    };
    const int slabs = (K + KL_SLAB - 1) / KL_SLAB;
    fetch(0);
    stage(0, 0);
    lds_barrier();
    for (int sl = 0; sl < slabs; ++sl) {
        const int buf = sl & 1;
        if (sl + 1 < slabs) fetch((sl + 1) * KL_SLAB);
        if (computes) {
            const bf16_t* base = lds + buf * KL_STAGE;
#pragma unroll
            for (int m = 0; m < 4; ++m) {
                kl_bf16x8 w[2], x[4];
#pragma unroll
                for (int wb = 0; wb < 2; ++wb)
                    w[wb] = *reinterpret_cast<const kl_bf16x8*>(base + (KL_ROWS + wave * 64 + wb * 32 + col) * KL_PITCH + half * 32 + m * 8);
#pragma unroll
                for (int rb = 0; rb < 4; ++rb)
                    x[rb] = *reinterpret_cast<const kl_bf16x8*>(base + (rb * 32 + col) * KL_PITCH + half * 32 + m * 8);
#pragma unroll
                for (int wb = 0; wb < 2; ++wb) {
                    if (MAY_SWAP && swap[wb]) {
#pragma unroll
                        for (int rb = 0; rb < 4; ++rb) acc[wb][rb] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(x[rb], w[wb], acc[wb][rb], 0, 0, 0);
                    } else {
#pragma unroll
                        for (int rb = 0; rb < 4; ++rb) acc[wb][rb] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(w[wb], x[rb], acc[wb][rb], 0, 0, 0);
                    }
                }
            }
        }
        if (sl + 1 < slabs) stage(buf ^ 1, (sl + 1) * KL_SLAB);
        lds_barrier();
    }
}
