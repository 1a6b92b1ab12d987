// Finishing a row of the fp32 residual stream: a sublayer's output d is normalised and added, x += d / rms(d) * gain with
// rms(d) = sqrt(mean(d^2) + eps), and the norm that the next reader of the stream begins with is computed from the new
// row, h = x / rms(x) * gain2, in the same pass. A workgroup of KA_ROW_THREADS threads takes a row; what computes d is the
// caller's business (a load, a weighted sum). All arithmetic is fp32.
#pragma once

#include "ka_common.h"

constexpr int KA_ROW_THREADS = 256;
constexpr int KA_ROW_WAVES = KA_ROW_THREADS / KA_WAVE;
constexpr int KA_ROW_MAX_PIECES = 8;        // pieces of four channels a thread keeps in registers: rows of up to 8192 channels

struct KaRowNorms {
    const float* gain;      // of the norm of d
    float eps;
    const float* gain2;     // of the norm of the new row; null: there is none
    float eps2;
    void* h;                // where that norm goes, rows of dim numbers
    int h_bf16;
};

__device__ __forceinline__ float ka_row_sum(float v, float* smem) {
    v = ka_wave_sum(v);
    __syncthreads();
    if (threadIdx.x % KA_WAVE == 0) smem[threadIdx.x / KA_WAVE] = v;
    __syncthreads();
    float total = 0.f;
#pragma unroll
    for (int w = 0; w < KA_ROW_WAVES; ++w) total += smem[w];
    return total;
}

__device__ __forceinline__ void ka_row_store_h(const KaRowNorms& a, size_t at, float v) {
    if (a.h_bf16) reinterpret_cast<bf16_t*>(a.h)[at] = (bf16_t)v;
    else reinterpret_cast<float*>(a.h)[at] = v;
}

// PIECES > 0: dim is a multiple of 4 and at most 4 PIECES KA_ROW_THREADS, rows are 16-byte aligned; `piece(c)` gives d of the
// channels c .. c + 3. PIECES = 0: any dim; `one(c)` gives d of channel c (asked for twice).
template <int PIECES, typename Piece, typename One>
__device__ __forceinline__ void ka_finish_row(float* __restrict__ x, int row, int dim, const KaRowNorms& a, Piece piece, One one,
                                              float* smem) {
    const int tid = threadIdx.x;
    const size_t at = (size_t)row * dim;
    if constexpr (PIECES > 0) {
        typedef __attribute__((ext_vector_type(4))) __bf16 row_bf16x4;
        float4 d[PIECES], y[PIECES];
        float s = 0.f;
#pragma unroll
        for (int p = 0; p < PIECES; ++p) {
            const int c = (p * KA_ROW_THREADS + tid) * 4;
            if (c < dim) {
                d[p] = piece(c);
                y[p] = *reinterpret_cast<const float4*>(x + at + c);
                s += d[p].x * d[p].x + d[p].y * d[p].y + d[p].z * d[p].z + d[p].w * d[p].w;
            }
        }
        const float r = 1.0f / sqrtf(ka_row_sum(s, smem) / (float)dim + a.eps);
        float s2 = 0.f;
#pragma unroll
        for (int p = 0; p < PIECES; ++p) {
            const int c = (p * KA_ROW_THREADS + tid) * 4;
            if (c < dim) {
                const float4 g = *reinterpret_cast<const float4*>(a.gain + c);
                y[p].x += d[p].x * r * g.x;
                y[p].y += d[p].y * r * g.y;
                y[p].z += d[p].z * r * g.z;
                y[p].w += d[p].w * r * g.w;
                *reinterpret_cast<float4*>(x + at + c) = y[p];
                s2 += y[p].x * y[p].x + y[p].y * y[p].y + y[p].z * y[p].z + y[p].w * y[p].w;
            }
        }
        if (a.gain2 == nullptr) return;
        const float r2 = 1.0f / sqrtf(ka_row_sum(s2, smem) / (float)dim + a.eps2);
#pragma unroll
        for (int p = 0; p < PIECES; ++p) {
            const int c = (p * KA_ROW_THREADS + tid) * 4;
            if (c < dim) {
                const float4 g = *reinterpret_cast<const float4*>(a.gain2 + c);
                const float4 v = make_float4(y[p].x * r2 * g.x, y[p].y * r2 * g.y, y[p].z * r2 * g.z, y[p].w * r2 * g.w);
                if (a.h_bf16) {
                    row_bf16x4 b;
                    b[0] = (bf16_t)v.x;
                    b[1] = (bf16_t)v.y;
                    b[2] = (bf16_t)v.z;
                    b[3] = (bf16_t)v.w;
                    *reinterpret_cast<row_bf16x4*>(reinterpret_cast<bf16_t*>(a.h) + at + c) = b;
                } else {
                    *reinterpret_cast<float4*>(reinterpret_cast<float*>(a.h) + at + c) = v;
                }
            }
        }
    } else {
        float s = 0.f;
        for (int c = tid; c < dim; c += KA_ROW_THREADS) {
            const float d = one(c);
            s += d * d;
        }
        const float r = 1.0f / sqrtf(ka_row_sum(s, smem) / (float)dim + a.eps);
        float s2 = 0.f;
        for (int c = tid; c < dim; c += KA_ROW_THREADS) {
            const float y = x[at + c] + one(c) * r * a.gain[c];
            x[at + c] = y;
            s2 += y * y;
        }
        if (a.gain2 == nullptr) return;
        const float r2 = 1.0f / sqrtf(ka_row_sum(s2, smem) / (float)dim + a.eps2);
        for (int c = tid; c < dim; c += KA_ROW_THREADS) ka_row_store_h(a, at + c, x[at + c] * r2 * a.gain2[c]);      // (its own writes)
    }
}

// Pieces of four channels a thread holds of rows of `dim` channels in the form with registers; 0: the general form.
static inline int ka_row_pieces(int dim, const void* x, const void* d, const KaRowNorms& a) {
    const uintptr_t all = (uintptr_t)x | (uintptr_t)d | (uintptr_t)a.gain | (uintptr_t)a.gain2;
    if (dim % 4 != 0 || all % 16 != 0 || (uintptr_t)a.h % (a.h_bf16 ? 8 : 16) != 0) return 0;
    const int need = (dim + 4 * KA_ROW_THREADS - 1) / (4 * KA_ROW_THREADS);
    for (int p : {1, 2, 4, 8})
        if (need <= p) return p;
    return 0;
}
