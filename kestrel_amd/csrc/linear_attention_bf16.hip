// Attention without a softmax over prompt portions on the matrix cores (bf16 operands, fp32 sums, fp32 state).
//
// The recurrence of a head, S_t = a S_(t-1) + v_t k_t^T, o_t = S_t q_t with one constant a = decay_h (S [dv, d]; see
// linear_attention.hip), is unrolled over a chunk of up to 64 tokens that starts from S_0 (tokens 0 .. L - 1 of the chunk):
//     o_t = sum_(s<=t) a^(t-s) (q_t . k_s) v_s + a^(t+1) S_0 q_t
//     S_L = a^L S_0 + sum_s a^(L-1-s) v_s k_s^T
// Every exponent is >= 0 and every power is computed by itself, 2^(n log2 a), so that no decay leaves its range.
// All chunks of a step are run at once, in three launches that meet in a buffer of the caller's (fp32, per chunk and head
// S [dv, d]): every chunk's state as if it started from nothing (LOCAL); a walk over a row's chunks, number by number in
// fp32, that turns those into the state every chunk starts from and advances the request's state (SCAN); every
// chunk's read-outs (READ).
//
// What is a sum over time or comes from the state enters its product as two bf16 numbers, the rounding and what it left
// (weighted values in LOCAL, weights and S_0 in READ): the products then keep sixteen bits of them, and a state is the
// same, but for the rounding of keys, however a sequence is cut. Queries and keys, and values where they are not weighted,
// are rounded to bf16 once, behind their activation. Workgroups of four waves own 64 value channels of a head; a value slice that ends before its 64
// channels, and a chunk that ends before its 64 tokens, is filled with zeros.
#include "ka_common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 lc_bf16x8;
typedef __attribute__((ext_vector_type(16))) float lc_floatx16;

constexpr int LC_CHUNK = 64;
constexpr int LC_SLICE = 64;                // value channels a workgroup
constexpr int LC_THREADS = 256;
constexpr int LC_PAD = 8;                   // elements an LDS row is longer than its data: spreads rows over the banks
constexpr int LC_ROW = LC_CHUNK + LC_PAD;
constexpr int LC_MAX_D = 256;

struct LinearChunkArgs {
    const bf16_t* q;
    const bf16_t* k;
    const bf16_t* v;
    long stride;
    const float* log2_decay;    // [H]
    float* state;               // [slots, state_stride]: S [H, dv, d]
    long state_stride;
    const int* cu_q;
    const int* row_slot;
    float* raw;                 // [n, H dv]
    float* chunks;              // [chunks, H, dv, d]
    int n_rows, H, d, dv, act;
};

// The row and the tokens [c0, c1) of chunk `g` of the step (chunks numbered row by row); false: behind the last chunk. A
// lane looks at a row, 64 rows at a time.
__device__ __forceinline__ bool lc_find_chunk(const LinearChunkArgs& a, int g, int& row, int& c0, int& c1) {
    const int lane = threadIdx.x % KA_WAVE;
    int base = 0;
    for (int r0 = 0; r0 < a.n_rows; r0 += KA_WAVE) {
        const int r = r0 + lane;
        const int t0 = r < a.n_rows ? a.cu_q[r] : 0, t1 = r < a.n_rows ? a.cu_q[r + 1] : 0;
        const int nc = (t1 - t0 + LC_CHUNK - 1) / LC_CHUNK;
        const int upto = base + (int)ka_wave_running_sum((float)nc);          // (counts of chunks: exact in fp32)
        const unsigned long long hit = __builtin_amdgcn_ballot_w64(g < upto && g >= upto - nc);
        if (hit != 0) {
            const int src = __builtin_ctzll(hit);
            row = r0 + src;
            const int first = __builtin_amdgcn_readlane(upto - nc, src);
            c0 = __builtin_amdgcn_readlane(t0, src) + (g - first) * LC_CHUNK;
            c1 = min(__builtin_amdgcn_readlane(t1, src), c0 + LC_CHUNK);
            return true;
        }
        base = __builtin_amdgcn_readlane(upto, KA_WAVE - 1);
    }
    return false;
}

__device__ __forceinline__ void lc_split(float x, bf16_t& hi, bf16_t& lo) {
    hi = (bf16_t)x;
    lo = (bf16_t)(x - (float)hi);
}

// LOCAL: S = sum_s a^(L-1-s) v_s k_s^T of one chunk and one slice of value channels. Grid (H, chunks, slices).
__global__ void __launch_bounds__(LC_THREADS) linear_chunk_local_kernel(LinearChunkArgs a) {
    extern __shared__ __attribute__((aligned(16))) bf16_t lc_lds[];
    int row, c0, c1;
    if (!lc_find_chunk(a, blockIdx.y, row, c0, c1)) return;
    if (a.row_slot[row] < 0) return;
    const int d = a.d, dv = a.dv, d32 = (d + 31) / 32 * 32;
    bf16_t* KT = lc_lds;                        // [d32][LC_ROW]: keys, channel by channel
    bf16_t* VH = KT + d32 * LC_ROW;             // [64][LC_ROW]: weighted values, channel by channel
    bf16_t* VL = VH + LC_SLICE * LC_ROW;        // what their rounding left
    const int head = blockIdx.x, tid = threadIdx.x, j0 = blockIdx.z * LC_SLICE;
    const int valid = c1 - c0;
    const float l2 = a.log2_decay[head];
    // (neighbouring lanes take neighbouring tokens: the transposed tiles are then written along their rows)
    for (int e = tid; e < LC_CHUNK * (d32 / 8); e += LC_THREADS) {
        const int t = e % LC_CHUNK, piece = e / LC_CHUNK;
        lc_bf16x8 x;
#pragma unroll
        for (int u = 0; u < 8; ++u) x[u] = (bf16_t)0.f;
        if (t < valid && piece * 8 < d) {
            x = *reinterpret_cast<const lc_bf16x8*>(a.k + (size_t)(c0 + t) * a.stride + (size_t)head * d + piece * 8);
#pragma unroll
            for (int u = 0; u < 8; ++u) x[u] = (bf16_t)ka_activate_fast(a.act, (float)x[u]);
        }
#pragma unroll
        for (int u = 0; u < 8; ++u) KT[(piece * 8 + u) * LC_ROW + t] = x[u];
    }
    for (int e = tid; e < LC_CHUNK * (LC_SLICE / 8); e += LC_THREADS) {
        const int t = e % LC_CHUNK, piece = e / LC_CHUNK;
        lc_bf16x8 hi, lo;
#pragma unroll
        for (int u = 0; u < 8; ++u) { hi[u] = (bf16_t)0.f; lo[u] = (bf16_t)0.f; }
        if (t < valid && j0 + piece * 8 < dv) {
            const lc_bf16x8 x = *reinterpret_cast<const lc_bf16x8*>(a.v + (size_t)(c0 + t) * a.stride + (size_t)head * dv + j0 + piece * 8);
            const float w = exp2f((float)(valid - 1 - t) * l2);
#pragma unroll
            for (int u = 0; u < 8; ++u) {
                bf16_t h, l;
                lc_split(ka_activate_fast(a.act, (float)x[u]) * w, h, l);
                hi[u] = h;
                lo[u] = l;
            }
        }
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            VH[(piece * 8 + u) * LC_ROW + t] = hi[u];
            VL[(piece * 8 + u) * LC_ROW + t] = lo[u];
        }
    }
    __syncthreads();
    const int wave = __builtin_amdgcn_readfirstlane(tid / KA_WAVE), lane = tid % KA_WAVE;
    const int col = lane % 32, half = lane / 32;
    const int jb = wave % 2;
    float* rec = a.chunks + ((size_t)blockIdx.y * a.H + head) * dv * d;
    for (int ib = wave / 2; ib < d32 / 32; ib += 2) {
        lc_floatx16 acc;
#pragma unroll
        for (int i = 0; i < 16; ++i) acc[i] = 0.f;
#pragma unroll
        for (int kk = 0; kk < LC_CHUNK; kk += 16) {
            const lc_bf16x8 kb = *reinterpret_cast<const lc_bf16x8*>(KT + (ib * 32 + col) * LC_ROW + kk + half * 8);
            acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const lc_bf16x8*>(VH + (jb * 32 + col) * LC_ROW + kk + half * 8), kb, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const lc_bf16x8*>(VL + (jb * 32 + col) * LC_ROW + kk + half * 8), kb, acc, 0, 0, 0);
        }
        // register i: value channel jb 32 + (i / 4) 8 + half 4 + i % 4, key channel ib 32 + col
        const int c = ib * 32 + col;
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const int j = j0 + jb * 32 + (i / 4) * 8 + half * 4 + i % 4;
            if (j < dv && c < d) rec[(size_t)j * d + c] = acc[i];
        }
    }
}

// SCAN: a row's chunks in order: every record gets the state its chunk starts from, the request's state is what the last
// chunk ends with. Grid (H, rows, slices of 1,024 numbers of S), four numbers a thread.
__global__ void __launch_bounds__(LC_THREADS) linear_chunk_scan_kernel(LinearChunkArgs a) {
    const int head = blockIdx.x, r = blockIdx.y, tid = threadIdx.x, lane = tid % KA_WAVE;
    const int t0 = a.cu_q[r], t1 = a.cu_q[r + 1];
    if (t0 >= t1) return;
    const int slot = a.row_slot[r];
    if (slot < 0) return;
    int before = 0;
    for (int q = lane; q < r; q += KA_WAVE) before += (a.cu_q[q + 1] - a.cu_q[q] + LC_CHUNK - 1) / LC_CHUNK;
    const int base = (int)ka_wave_sum((float)before);
    const int nc = (t1 - t0 + LC_CHUNK - 1) / LC_CHUNK;
    const int per = a.d * a.dv;
    const int e = (blockIdx.z * LC_THREADS + tid) * 4;
    if (e >= per) return;
    float* st = a.state + (size_t)slot * a.state_stride + (size_t)head * per + e;
    float* rec = a.chunks + ((size_t)base * a.H + head) * per + e;
    const size_t step = (size_t)a.H * per;
    const float l2 = a.log2_decay[head];
    const float whole = exp2f((float)LC_CHUNK * l2), last = exp2f((float)(t1 - t0 - (nc - 1) * LC_CHUNK) * l2);
    float4 cur = *reinterpret_cast<const float4*>(st);
    auto advance = [&](float f, const float4& x) {
        cur.x = fmaf(f, cur.x, x.x);
        cur.y = fmaf(f, cur.y, x.y);
        cur.z = fmaf(f, cur.z, x.z);
        cur.w = fmaf(f, cur.w, x.w);
    };
    int c = 0;
    for (; c + 8 < nc; c += 8) {                // (eight records in flight; the last chunk is taken below)
        float4 x[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) x[u] = *reinterpret_cast<const float4*>(rec + (c + u) * step);
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            *reinterpret_cast<float4*>(rec + (c + u) * step) = cur;
            advance(whole, x[u]);
        }
    }
    for (; c < nc; ++c) {
        const float4 x = *reinterpret_cast<const float4*>(rec + c * step);
        *reinterpret_cast<float4*>(rec + c * step) = cur;
        advance(c + 1 < nc ? whole : last, x);
    }
    *reinterpret_cast<float4*>(st) = cur;
}

// READ: the read-outs of one chunk and one slice of value channels. Wave w takes the tokens [32 (w % 2), + 32) and the value
// channels [32 (w / 2), + 32). Scores are computed transposed, keys as the row operand with bits 2 and 3 of the row index
// swapped, so that the eight weights a lane holds are those of eight consecutive keys of its token: as they stand, the
// column operand of the product with the values. Grid (H, chunks, slices).
__global__ void __launch_bounds__(LC_THREADS) linear_chunk_read_kernel(LinearChunkArgs a) {
    extern __shared__ __attribute__((aligned(16))) bf16_t lc_lds[];
    int row, c0, c1;
    if (!lc_find_chunk(a, blockIdx.y, row, c0, c1)) return;
    const int d = a.d, dv = a.dv, lq = d + LC_PAD;
    const int head = blockIdx.x, tid = threadIdx.x, j0 = blockIdx.z * LC_SLICE;
    const int valid = c1 - c0;
    const size_t out_row = (size_t)a.H * dv;
    if (a.row_slot[row] < 0) {
        for (int e = tid; e < valid * LC_SLICE; e += LC_THREADS)
            if (j0 + e % LC_SLICE < dv) a.raw[(size_t)(c0 + e / LC_SLICE) * out_row + (size_t)head * dv + j0 + e % LC_SLICE] = 0.f;
        return;
    }
    bf16_t* Qs = lc_lds;                        // [64][lq]
    bf16_t* Ks = Qs + LC_CHUNK * lq;            // [64][lq]
    bf16_t* VT = Ks + LC_CHUNK * lq;            // [64][LC_ROW]: values, channel by channel
    const int pieces = d / 8;
    for (int e = tid; e < LC_CHUNK * pieces; e += LC_THREADS) {
        const int t = e / pieces, piece = e % pieces;
        lc_bf16x8 q, k;
#pragma unroll
        for (int u = 0; u < 8; ++u) { q[u] = (bf16_t)0.f; k[u] = (bf16_t)0.f; }
        if (t < valid) {
            const size_t at = (size_t)(c0 + t) * a.stride + (size_t)head * d + piece * 8;
            q = *reinterpret_cast<const lc_bf16x8*>(a.q + at);
            k = *reinterpret_cast<const lc_bf16x8*>(a.k + at);
#pragma unroll
            for (int u = 0; u < 8; ++u) {
                q[u] = (bf16_t)ka_activate_fast(a.act, (float)q[u]);
                k[u] = (bf16_t)ka_activate_fast(a.act, (float)k[u]);
            }
        }
        *reinterpret_cast<lc_bf16x8*>(Qs + t * lq + piece * 8) = q;
        *reinterpret_cast<lc_bf16x8*>(Ks + t * lq + piece * 8) = k;
    }
    for (int e = tid; e < LC_CHUNK * (LC_SLICE / 8); e += LC_THREADS) {
        const int t = e % LC_CHUNK, piece = e / LC_CHUNK;
        lc_bf16x8 x;
#pragma unroll
        for (int u = 0; u < 8; ++u) x[u] = (bf16_t)0.f;
        if (t < valid && j0 + piece * 8 < dv) {
            x = *reinterpret_cast<const lc_bf16x8*>(a.v + (size_t)(c0 + t) * a.stride + (size_t)head * dv + j0 + piece * 8);
#pragma unroll
            for (int u = 0; u < 8; ++u) x[u] = (bf16_t)ka_activate_fast(a.act, (float)x[u]);
        }
#pragma unroll
        for (int u = 0; u < 8; ++u) VT[(piece * 8 + u) * LC_ROW + t] = x[u];
    }
    __syncthreads();
    const int wave = __builtin_amdgcn_readfirstlane(tid / KA_WAVE), lane = tid % KA_WAVE;
    const int col = lane % 32, half = lane / 32;
    const int tb = wave % 2, jb = wave / 2;
    if (tb * 32 >= valid || j0 + jb * 32 >= dv) return;           // (no barrier behind this)
    const float l2 = a.log2_decay[head];
    const int t = tb * 32 + col;
    // S_0 q_t, then the power of the decay that belongs to the lane's token
    lc_floatx16 o;
#pragma unroll
    for (int i = 0; i < 16; ++i) o[i] = 0.f;
    const float* srow = a.chunks + ((size_t)blockIdx.y * a.H + head) * dv * d + (size_t)min(j0 + jb * 32 + col, dv - 1) * d + half * 8;
    for (int kk = 0; kk < d; kk += 16) {
        const float4 s0 = *reinterpret_cast<const float4*>(srow + kk), s1 = *reinterpret_cast<const float4*>(srow + kk + 4);
        const float x[8] = {s0.x, s0.y, s0.z, s0.w, s1.x, s1.y, s1.z, s1.w};
        lc_bf16x8 hi, lo;
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            bf16_t h, l;
            lc_split(x[u], h, l);
            hi[u] = h;
            lo[u] = l;
        }
        const lc_bf16x8 qb = *reinterpret_cast<const lc_bf16x8*>(Qs + t * lq + kk + half * 8);
        o = __builtin_amdgcn_mfma_f32_32x32x16_bf16(hi, qb, o, 0, 0, 0);
        o = __builtin_amdgcn_mfma_f32_32x32x16_bf16(lo, qb, o, 0, 0, 0);
    }
    const float carried = exp2f((float)(t + 1) * l2);
#pragma unroll
    for (int i = 0; i < 16; ++i) o[i] *= carried;
    const int krow = (col & 0x13) | ((col & 4) << 1) | ((col & 8) >> 1);
    for (int sb = 0; sb <= tb; ++sb) {
        lc_floatx16 g;
#pragma unroll
        for (int i = 0; i < 16; ++i) g[i] = 0.f;
        for (int kk = 0; kk < d; kk += 16)
            g = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const lc_bf16x8*>(Ks + (sb * 32 + krow) * lq + kk + half * 8),
                                                        *reinterpret_cast<const lc_bf16x8*>(Qs + t * lq + kk + half * 8), g, 0, 0, 0);
        lc_bf16x8 ph[2], pl[2];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            // register i: key sb 32 + (i / 8) 16 + half 8 + i % 8 of the lane's token
            const int s = sb * 32 + (i / 8) * 16 + half * 8 + i % 8;
            const float p = s <= t ? g[i] * exp2f((float)(t - s) * l2) : 0.f;
            bf16_t h, l;
            lc_split(p, h, l);
            ph[i / 8][i % 8] = h;
            pl[i / 8][i % 8] = l;
        }
#pragma unroll
        for (int p = 0; p < 2; ++p) {
            const lc_bf16x8 va = *reinterpret_cast<const lc_bf16x8*>(VT + (jb * 32 + col) * LC_ROW + sb * 32 + p * 16 + half * 8);
            o = __builtin_amdgcn_mfma_f32_32x32x16_bf16(va, ph[p], o, 0, 0, 0);
            o = __builtin_amdgcn_mfma_f32_32x32x16_bf16(va, pl[p], o, 0, 0, 0);
        }
    }
    if (t >= valid) return;
    float* op = a.raw + (size_t)(c0 + t) * out_row + (size_t)head * dv + j0 + jb * 32;
#pragma unroll
    for (int g4 = 0; g4 < 4; ++g4) {
        const int j = g4 * 8 + half * 4;
        if (j0 + jb * 32 + j < dv) *reinterpret_cast<float4*>(op + j) = make_float4(o[g4 * 4], o[g4 * 4 + 1], o[g4 * 4 + 2], o[g4 * 4 + 3]);
    }
}

// Whether the kernels cover heads of these sizes: keys in steps of 16 up to 256 channels, values in steps of 8.
KA_API int ka_linear_chunks_supported(int d, int dv) { return d > 0 && d % 16 == 0 && d <= LC_MAX_D && dv > 0 && dv % 8 == 0 ? 1 : 0; }

// Chunks, and floats of the launches' buffer, of a step of `n` tokens in `n_rows` rows (every row may end in a part of a chunk).
KA_API long ka_linear_chunks_scratch(int n, int n_rows, int H, int d, int dv) { return (long)(n / LC_CHUNK + n_rows) * H * d * dv; }

KA_API int ka_linear_chunks_bf16(const void* q, const void* k, const void* v, long stride, const float* log2_decay, float* state,
                                 long state_stride, const int* cu_q, const int* row_slot, float* raw, float* chunks, int n, int n_rows,
                                 int H, int d, int dv, int act, hipStream_t stream) {
    const char* who = "ka_linear_chunks_bf16";
    KA_CHECK(n >= 0 && n_rows >= 0 && H > 0 && ka_linear_chunks_supported(d, dv), "%s: heads of %d x %d not covered", who, d, dv);
    KA_CHECK(ka_act_known(act) && !ka_act_gated(act), "%s: unknown activation %d", who, act);
    KA_CHECK((uintptr_t)q % 16 == 0 && (uintptr_t)k % 16 == 0 && (uintptr_t)v % 16 == 0 && stride % 8 == 0 && (uintptr_t)raw % 16 == 0 &&
             (uintptr_t)chunks % 16 == 0 && (uintptr_t)state % 16 == 0 && state_stride % 4 == 0, "%s: operands must be 16-byte aligned", who);
    KA_CHECK(state_stride >= (long)H * d * dv && stride >= (long)H * d && stride >= (long)H * dv, "%s: rows are shorter than their heads", who);
    const long n_chunks = n / LC_CHUNK + n_rows;
    KA_CHECK(H <= 65535 && n_rows <= 65535 && n_chunks <= 65535 && chunks != nullptr, "%s: too many heads, rows or chunks", who);
    if (n == 0 || n_rows == 0) return 0;
    LinearChunkArgs a{(const bf16_t*)q, (const bf16_t*)k, (const bf16_t*)v, stride, log2_decay, state, state_stride, cu_q, row_slot, raw,
                      chunks, n_rows, H, d, dv, act};
    const int slices = ka_cdiv(dv, LC_SLICE), d32 = (d + 31) / 32 * 32;
    const size_t local_lds = sizeof(bf16_t) * (size_t)(d32 + 2 * LC_SLICE) * LC_ROW;
    const size_t read_lds = sizeof(bf16_t) * ((size_t)2 * LC_CHUNK * (d + LC_PAD) + (size_t)LC_SLICE * LC_ROW);
    static bool sized = false;
    if (!sized) {
        (void)hipFuncSetAttribute((const void*)linear_chunk_local_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
        (void)hipFuncSetAttribute((const void*)linear_chunk_read_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
        sized = true;
    }
    hipLaunchKernelGGL(linear_chunk_local_kernel, dim3(H, n_chunks, slices), dim3(LC_THREADS), local_lds, stream, a);
    hipLaunchKernelGGL(linear_chunk_scan_kernel, dim3(H, n_rows, ka_cdiv((long)d * dv, 4 * LC_THREADS)), dim3(LC_THREADS), 0, stream, a);
    hipLaunchKernelGGL(linear_chunk_read_kernel, dim3(H, n_chunks, slices), dim3(LC_THREADS), read_lds, stream, a);
    KA_LAUNCH_CHECK();
    return 0;
}
