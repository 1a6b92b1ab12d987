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
//
// The same three launches serve a recurrence that forgets key channel by key channel, by factors computed from the tokens
// (further below).
#include "ka_common.h"
#include "ka_decay.h"

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
// chunk ends with. Grid (H, rows, slices of 1,024 numbers of S), four numbers a thread. BY_CHANNEL: what a chunk's state keeps of
// the one before comes from `factors` [chunks, H, d], key channel by key channel.
template <bool BY_CHANNEL>
__global__ void __launch_bounds__(LC_THREADS) linear_chunk_scan_kernel(LinearChunkArgs a, const float* __restrict__ factors) {
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
    const float l2 = BY_CHANNEL ? 0.f : a.log2_decay[head];
    const float whole = exp2f((float)LC_CHUNK * l2), last = exp2f((float)(t1 - t0 - (nc - 1) * LC_CHUNK) * l2);
    // (the four numbers are of four neighbouring key channels)
    const float* fac = BY_CHANNEL ? factors + ((size_t)base * a.H + head) * a.d + e % a.d : nullptr;
    auto kept = [&](int c) {
        if constexpr (BY_CHANNEL) return *reinterpret_cast<const float4*>(fac + (size_t)c * a.H * a.d);
        const float f = c + 1 < nc ? whole : last;
        return make_float4(f, f, f, f);
    };
    float4 cur = *reinterpret_cast<const float4*>(st);
    auto advance = [&](const float4& f, const float4& x) {
        cur.x = fmaf(f.x, cur.x, x.x);
        cur.y = fmaf(f.y, cur.y, x.y);
        cur.z = fmaf(f.z, cur.z, x.z);
        cur.w = fmaf(f.w, cur.w, x.w);
    };
    int c = 0;
    for (; c + 8 < nc; c += 8) {                // (eight records in flight; the last chunk is taken below)
        float4 x[8], f[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            x[u] = *reinterpret_cast<const float4*>(rec + (c + u) * step);
            f[u] = kept(c + u);
        }
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            *reinterpret_cast<float4*>(rec + (c + u) * step) = cur;
            advance(f[u], x[u]);
        }
    }
    for (; c < nc; ++c) {
        const float4 x = *reinterpret_cast<const float4*>(rec + c * step), f = kept(c);
        *reinterpret_cast<float4*>(rec + c * step) = cur;
        advance(f, x);
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
    hipLaunchKernelGGL(linear_chunk_scan_kernel<false>, dim3(H, n_rows, ka_cdiv((long)d * dv, 4 * LC_THREADS)), dim3(LC_THREADS), 0, stream, a, nullptr);
    hipLaunchKernelGGL(linear_chunk_read_kernel, dim3(H, n_chunks, slices), dim3(LC_THREADS), read_lds, stream, a);
    KA_LAUNCH_CHECK();
    return 0;
}

// ----------------------------------------------------------------------------
// A recurrence that forgets channel by channel: S_t = S_(t-1) diag(a_t) + v_t k_t^T, o_t = S_t (q_scale q_t), with a factor
// a_t[i] = sigmoid(pre_t[i])^(1 / tau) per token and key channel (ka_decay.h). With b_t[i] the sum of log2 a_r[i] over the chunk's
// tokens r <= t:
//     o_t = q_scale (sum_(s<=t) (sum_i q_t[i] k_s[i] 2^(b_t[i] - b_s[i])) v_s + sum_i q_t[i] 2^(b_t[i]) S_0[:, i])
//     S_L[:, i] = 2^(b_L[i]) S_0[:, i] + sum_s 2^(b_L[i] - b_s[i]) k_s[i] v_s
// The powers do not leave the sum over i. A chunk is cut into four blocks of 16 tokens, and sums of logarithms are kept from a
// block's start, l_t, and up to it, B_T (b_t = B_T + l_t). Between blocks U < T a score is the product of q_t 2^(l_t) and
// k_s 2^(B_T - b_s), both powers at most 1, on the matrix cores; within a block every power is taken by itself. So no factor,
// however small, leaves its range. What carries a power enters its product as two bf16 numbers, as above.
// ----------------------------------------------------------------------------
constexpr int LC_BLOCK = 16;
constexpr int LC_BLOCKS = LC_CHUNK / LC_BLOCK;
constexpr int LC_GATED_MAX_D = 224;

typedef __attribute__((ext_vector_type(4))) float lc_floatx4;
typedef __attribute__((ext_vector_type(4))) __bf16 lc_bf16x4;

struct GatedChunkArgs : LinearChunkArgs {
    const float* pre;           // [n, H d]
    float* factors;             // [chunks, H, d]: 2^(b_L) of every chunk
    float per_tau, q_scale;     // 1 / tau
};

__device__ __forceinline__ float lc_exp2(float x) { return __builtin_amdgcn_exp2f(x); }

// Values of the chunk, channel by channel: VT [64][LC_ROW], zeros behind the last token and the last channel.
__device__ __forceinline__ void lc_stage_values(const LinearChunkArgs& a, bf16_t* VT, int head, int c0, int valid, int j0) {
    for (int e = threadIdx.x; e < LC_CHUNK * (LC_SLICE / 8); e += LC_THREADS) {
        const int t = e % LC_CHUNK, piece = e / LC_CHUNK;
        lc_bf16x8 x;
#pragma unroll
        for (int u = 0; u < 8; ++u) x[u] = (bf16_t)0.f;
        if (t < valid && j0 + piece * 8 < a.dv)
            x = *reinterpret_cast<const lc_bf16x8*>(a.v + (size_t)(c0 + t) * a.stride + (size_t)head * a.dv + j0 + piece * 8);
#pragma unroll
        for (int u = 0; u < 8; ++u) VT[(piece * 8 + u) * LC_ROW + t] = x[u];
    }
}

// l of the 16 tokens of block `block` for key channel i of the head (zeros behind the last token and the last channel).
__device__ __forceinline__ void lc_block_logs(const GatedChunkArgs& a, int head, int c0, int valid, int block, int i, float (&l)[LC_BLOCK]) {
    const float* z = a.pre + (size_t)c0 * a.H * a.d + (size_t)head * a.d + i;
    float x[LC_BLOCK];
#pragma unroll
    for (int u = 0; u < LC_BLOCK; ++u) {
        const int t = block * LC_BLOCK + u;
        x[u] = i < a.d && t < valid ? z[(size_t)t * a.H * a.d] : 0.f;
    }
    float run = 0.f;
#pragma unroll
    for (int u = 0; u < LC_BLOCK; ++u) {
        if (i < a.d && block * LC_BLOCK + u < valid) run += ka_log2_decay<true>(x[u], a.per_tau);
        l[u] = run;
    }
}

// LOCAL: what the chunk adds to the state by its end, of one slice of value channels, and (the first slice) its factors.
// Grid (H, chunks, slices). A wave takes a block of tokens, a lane a key channel.
__global__ void __launch_bounds__(LC_THREADS) gated_chunk_local_kernel(GatedChunkArgs a) {
    extern __shared__ __attribute__((aligned(16))) bf16_t lc_lds[];
    int row, c0, c1;
    if (!lc_find_chunk(a, blockIdx.y, row, c0, c1)) return;
    if (a.row_slot[row] < 0) return;
    const int d = a.d, dv = a.dv, d32 = (d + 31) / 32 * 32, d64 = (d + 63) / 64 * 64;
    bf16_t* KH = lc_lds;                        // [d32][LC_ROW]: weighted keys, channel by channel
    bf16_t* KL = KH + d32 * LC_ROW;             // what their rounding left
    bf16_t* VT = KL + d32 * LC_ROW;             // [64][LC_ROW]: values, channel by channel
    float* sums = reinterpret_cast<float*>(VT + LC_SLICE * LC_ROW);      // [4][d64]: l at every block's end
    const int head = blockIdx.x, tid = threadIdx.x, j0 = blockIdx.z * LC_SLICE;
    const int valid = c1 - c0;
    const int wave = __builtin_amdgcn_readfirstlane(tid / KA_WAVE), lane = tid % KA_WAVE;
    lc_stage_values(a, VT, head, c0, valid, j0);
    for (int i = lane; i < d64; i += KA_WAVE) {
        float l[LC_BLOCK];
        lc_block_logs(a, head, c0, valid, wave, i, l);
        bf16_t k[LC_BLOCK];
#pragma unroll
        for (int u = 0; u < LC_BLOCK; ++u) {
            const int t = wave * LC_BLOCK + u;
            k[u] = i < d && t < valid ? a.k[(size_t)(c0 + t) * a.stride + (size_t)head * d + i] : (bf16_t)0.f;
        }
        sums[wave * d64 + i] = l[LC_BLOCK - 1];
        __syncthreads();
        float all = 0.f, upto = 0.f;            // (up to this block's end)
#pragma unroll
        for (int b = 0; b < LC_BLOCKS; ++b) {
            all += sums[b * d64 + i];
            if (b <= wave) upto += sums[b * d64 + i];
        }
        if (wave == 0 && i < d && blockIdx.z == 0) a.factors[((size_t)blockIdx.y * a.H + head) * d + i] = lc_exp2(all);
        if (i < d32) {
#pragma unroll
            for (int half = 0; half < 2; ++half) {
                lc_bf16x8 hi, lo;
#pragma unroll
                for (int u = 0; u < 8; ++u) {
                    bf16_t h, r;
                    lc_split((float)k[half * 8 + u] * lc_exp2((all - upto) + (l[LC_BLOCK - 1] - l[half * 8 + u])), h, r);
                    hi[u] = h;
                    lo[u] = r;
                }
                *reinterpret_cast<lc_bf16x8*>(KH + i * LC_ROW + wave * LC_BLOCK + half * 8) = hi;
                *reinterpret_cast<lc_bf16x8*>(KL + i * LC_ROW + wave * LC_BLOCK + half * 8) = lo;
            }
        }
    }
    __syncthreads();
    const int col = lane % 32, half = lane / 32;
    const int jb = wave % 2;
    if (j0 + jb * 32 >= dv) return;             // (no barrier behind this)
    float* rec = a.chunks + ((size_t)blockIdx.y * a.H + head) * dv * d;
    for (int ib = wave / 2; ib < d32 / 32; ib += 2) {
        lc_floatx16 acc;
#pragma unroll
        for (int i = 0; i < 16; ++i) acc[i] = 0.f;
#pragma unroll
        for (int kk = 0; kk < LC_CHUNK; kk += 16) {
            const lc_bf16x8 va = *reinterpret_cast<const lc_bf16x8*>(VT + (jb * 32 + col) * LC_ROW + kk + half * 8);
            acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(va, *reinterpret_cast<const lc_bf16x8*>(KH + (ib * 32 + col) * LC_ROW + kk + half * 8), acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(va, *reinterpret_cast<const lc_bf16x8*>(KL + (ib * 32 + col) * LC_ROW + kk + half * 8), acc, 0, 0, 0);
        }
        const int c = ib * 32 + col;
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const int j = j0 + jb * 32 + (i / 4) * 8 + half * 4 + i % 4;
            if (j < dv && c < d) rec[(size_t)j * d + c] = acc[i];
        }
    }
}

// READ: the read-outs of one chunk. Wave T takes the queries of block T. Grid (H, chunks, value slices at once); a workgroup
// takes every gridDim.z-th slice of 64 value channels. In all products the queries are the column operand: a lane ends with
// results of one query.
__global__ void __launch_bounds__(LC_THREADS) gated_chunk_read_kernel(GatedChunkArgs a) {
    extern __shared__ __attribute__((aligned(16))) bf16_t lc_lds[];
    int row, c0, c1;
    if (!lc_find_chunk(a, blockIdx.y, row, c0, c1)) return;
    const int d = a.d, dv = a.dv, d32 = (d + 31) / 32 * 32, lq = d32 + LC_PAD, lb = d32 + 4;
    const int head = blockIdx.x, tid = threadIdx.x;
    const int valid = c1 - c0;
    const size_t out_row = (size_t)a.H * dv;
    if (a.row_slot[row] < 0) {
        if (blockIdx.z == 0)
            for (int e = tid; e < valid * dv; e += LC_THREADS) a.raw[(size_t)(c0 + e / dv) * out_row + (size_t)head * dv + e % dv] = 0.f;
        return;
    }
    bf16_t* Qs = lc_lds;                        // [64][lq]
    bf16_t* Ks = Qs + LC_CHUNK * lq;            // [64][lq]
    bf16_t* VT = Ks + LC_CHUNK * lq;            // [64][LC_ROW]
    bf16_t* PH = VT + LC_SLICE * LC_ROW;        // [64][LC_ROW]: scores, query by query
    bf16_t* PL = PH + LC_CHUNK * LC_ROW;        // what their rounding left
    float* Ls = reinterpret_cast<float*>(PL + LC_CHUNK * LC_ROW);        // [64][lb]: l
    float* Bs = Ls + LC_CHUNK * lb;             // [4][d32]: B
    const int wave = __builtin_amdgcn_readfirstlane(tid / KA_WAVE), lane = tid % KA_WAVE;
    const int pieces = d32 / 8;
    for (int e = tid; e < LC_CHUNK * pieces; e += LC_THREADS) {
        const int t = e / pieces, piece = e % pieces;
        lc_bf16x8 q, k;
#pragma unroll
        for (int u = 0; u < 8; ++u) { q[u] = (bf16_t)0.f; k[u] = (bf16_t)0.f; }
        if (t < valid && piece * 8 < d) {
            const size_t at = (size_t)(c0 + t) * a.stride + (size_t)head * d + piece * 8;
            q = *reinterpret_cast<const lc_bf16x8*>(a.q + at);
            k = *reinterpret_cast<const lc_bf16x8*>(a.k + at);
        }
        *reinterpret_cast<lc_bf16x8*>(Qs + t * lq + piece * 8) = q;
        *reinterpret_cast<lc_bf16x8*>(Ks + t * lq + piece * 8) = k;
    }
    for (int i = lane; i < d32; i += KA_WAVE) {
        float l[LC_BLOCK];
        lc_block_logs(a, head, c0, valid, wave, i, l);
#pragma unroll
        for (int u = 0; u < LC_BLOCK; ++u) Ls[(wave * LC_BLOCK + u) * lb + i] = l[u];
    }
    __syncthreads();
    for (int i = tid; i < d32; i += LC_THREADS) {
        float upto = 0.f;
#pragma unroll
        for (int b = 0; b < LC_BLOCKS; ++b) {
            Bs[b * d32 + i] = upto;
            upto += Ls[(b * LC_BLOCK + LC_BLOCK - 1) * lb + i];
        }
    }
    __syncthreads();
    const int col = lane % 16, quarter = lane / 16;
    const bool active = wave * LC_BLOCK < valid;
    const int t = wave * LC_BLOCK + col;        // the lane's query (and, within the block, the lane's key)
    // q_t 2^(l_t) of the eight channels from c on
    auto query = [&](int c, lc_bf16x8& hi, lc_bf16x8& lo) {
        const lc_bf16x8 x = *reinterpret_cast<const lc_bf16x8*>(Qs + t * lq + c);
        const lc_floatx4 l0 = *reinterpret_cast<const lc_floatx4*>(Ls + t * lb + c), l1 = *reinterpret_cast<const lc_floatx4*>(Ls + t * lb + c + 4);
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            bf16_t h, r;
            lc_split((float)x[u] * a.q_scale * lc_exp2(u < 4 ? l0[u % 4] : l1[u % 4]), h, r);
            hi[u] = h;
            lo[u] = r;
        }
    };
    if (active) {
        // within the block: the lane's key, a quarter of the channels, all queries
        float score[LC_BLOCK];
#pragma unroll
        for (int u = 0; u < LC_BLOCK; ++u) score[u] = 0.f;
        for (int c = quarter * (d32 / 4); c < (quarter + 1) * (d32 / 4); c += 8) {
            const lc_bf16x8 k = *reinterpret_cast<const lc_bf16x8*>(Ks + t * lq + c);
            const lc_floatx4 k0 = *reinterpret_cast<const lc_floatx4*>(Ls + t * lb + c), k1 = *reinterpret_cast<const lc_floatx4*>(Ls + t * lb + c + 4);
#pragma unroll
            for (int u = 0; u < LC_BLOCK; ++u) {
                const int at = wave * LC_BLOCK + u;
                const lc_bf16x8 q = *reinterpret_cast<const lc_bf16x8*>(Qs + at * lq + c);
                const lc_floatx4 l0 = *reinterpret_cast<const lc_floatx4*>(Ls + at * lb + c), l1 = *reinterpret_cast<const lc_floatx4*>(Ls + at * lb + c + 4);
#pragma unroll
                for (int m = 0; m < 8; ++m) {
                    const float gap = m < 4 ? l0[m % 4] - k0[m % 4] : l1[m % 4] - k1[m % 4];
                    score[u] = fmaf((float)q[m] * (float)k[m], lc_exp2(fminf(gap, 0.f)), score[u]);      // (keys behind their query: not used)
                }
            }
        }
#pragma unroll
        for (int u = 0; u < LC_BLOCK; ++u) {
            float s = score[u];
            s += __shfl_xor(s, 16);
            s += __shfl_xor(s, 32);
            if (quarter == u % 4) {
                bf16_t h, r;
                lc_split(col <= u ? s * a.q_scale : 0.f, h, r);
                PH[(wave * LC_BLOCK + u) * LC_ROW + t] = h;
                PL[(wave * LC_BLOCK + u) * LC_ROW + t] = r;
            }
        }
        // the blocks before it
        lc_floatx4 g[LC_BLOCKS - 1];
#pragma unroll
        for (int b = 0; b < LC_BLOCKS - 1; ++b) g[b] = lc_floatx4{0.f, 0.f, 0.f, 0.f};
        if (wave > 0) {
            for (int kk = 0; kk < d32; kk += 32) {
                const int c = kk + quarter * 8;
                lc_bf16x8 qh, ql;
                query(c, qh, ql);
                const float* to = Bs + wave * d32 + c;
#pragma unroll
                for (int b = 0; b < LC_BLOCKS - 1; ++b) {
                    if (b >= wave) continue;
                    const int s = b * LC_BLOCK + col;
                    const lc_bf16x8 x = *reinterpret_cast<const lc_bf16x8*>(Ks + s * lq + c);
                    lc_bf16x8 kh, kl;
#pragma unroll
                    for (int u = 0; u < 8; ++u) {
                        bf16_t h, r;
                        lc_split((float)x[u] * lc_exp2(to[u] - Bs[b * d32 + c + u] - Ls[s * lb + c + u]), h, r);
                        kh[u] = h;
                        kl[u] = r;
                    }
                    g[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kh, qh, g[b], 0, 0, 0);
                    g[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kl, qh, g[b], 0, 0, 0);
                    g[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kh, ql, g[b], 0, 0, 0);
                }
            }
        }
        // (keys are taken 32 at a time below: the block behind an even one is zero)
#pragma unroll
        for (int b = 0; b < LC_BLOCKS; ++b) {
            if (!(b < wave || (b == wave + 1 && wave % 2 == 0))) continue;
            lc_bf16x4 hi, lo;
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                bf16_t h, r;
                lc_split(b < wave ? g[b < LC_BLOCKS - 1 ? b : 0][u] : 0.f, h, r);
                hi[u] = h;
                lo[u] = r;
            }
            *reinterpret_cast<lc_bf16x4*>(PH + t * LC_ROW + b * LC_BLOCK + quarter * 4) = hi;
            *reinterpret_cast<lc_bf16x4*>(PL + t * LC_ROW + b * LC_BLOCK + quarter * 4) = lo;
        }
    }
    const float* S0 = a.chunks + ((size_t)blockIdx.y * a.H + head) * dv * d;
    for (int j0 = blockIdx.z * LC_SLICE; j0 < dv; j0 += gridDim.z * LC_SLICE) {
        __syncthreads();
        lc_stage_values(a, VT, head, c0, valid, j0);
        __syncthreads();
        if (!active) continue;
        lc_floatx4 o[LC_SLICE / 16];
#pragma unroll
        for (int j = 0; j < LC_SLICE / 16; ++j) o[j] = lc_floatx4{0.f, 0.f, 0.f, 0.f};
        for (int kk = 0; kk < d32; kk += 32) {
            const int c = kk + quarter * 8;
            lc_bf16x8 qh, ql;
            query(c, qh, ql);
            float upto[8];
#pragma unroll
            for (int u = 0; u < 8; ++u) upto[u] = c < d ? lc_exp2(Bs[wave * d32 + c + u]) : 0.f;
#pragma unroll
            for (int j = 0; j < LC_SLICE / 16; ++j) {
                if (j0 + j * 16 >= dv) continue;
                const float* srow = S0 + (size_t)min(j0 + j * 16 + col, dv - 1) * d + min(c, d - 8);
                const lc_floatx4 s0 = *reinterpret_cast<const lc_floatx4*>(srow), s1 = *reinterpret_cast<const lc_floatx4*>(srow + 4);
                lc_bf16x8 hi, lo;
#pragma unroll
                for (int u = 0; u < 8; ++u) {
                    bf16_t h, r;
                    lc_split((u < 4 ? s0[u % 4] : s1[u % 4]) * upto[u], h, r);
                    hi[u] = h;
                    lo[u] = r;
                }
                o[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi, qh, o[j], 0, 0, 0);
                o[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo, qh, o[j], 0, 0, 0);
                o[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi, ql, o[j], 0, 0, 0);
            }
        }
        for (int sb = 0; sb <= wave / 2; ++sb) {
            const lc_bf16x8 ph = *reinterpret_cast<const lc_bf16x8*>(PH + t * LC_ROW + sb * 32 + quarter * 8);
            const lc_bf16x8 pl = *reinterpret_cast<const lc_bf16x8*>(PL + t * LC_ROW + sb * 32 + quarter * 8);
#pragma unroll
            for (int j = 0; j < LC_SLICE / 16; ++j) {
                const lc_bf16x8 va = *reinterpret_cast<const lc_bf16x8*>(VT + (j * 16 + col) * LC_ROW + sb * 32 + quarter * 8);
                o[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(va, ph, o[j], 0, 0, 0);
                o[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(va, pl, o[j], 0, 0, 0);
            }
        }
        if (t >= valid) continue;
        float* op = a.raw + (size_t)(c0 + t) * out_row + (size_t)head * dv + j0 + quarter * 4;
#pragma unroll
        for (int j = 0; j < LC_SLICE / 16; ++j)
            if (j0 + j * 16 + quarter * 4 < dv) *reinterpret_cast<lc_floatx4*>(op + j * 16) = o[j];
    }
}

// Whether the kernels cover heads of these sizes: keys in steps of 16 up to 224 channels, values in steps of 8.
KA_API int ka_gated_chunks_supported(int d, int dv) { return d > 0 && d % 16 == 0 && d <= LC_GATED_MAX_D && dv > 0 && dv % 8 == 0 ? 1 : 0; }

// Floats of the launches' buffer of a step of `n` tokens in `n_rows` rows: a state and its factors per chunk and head.
KA_API long ka_gated_chunks_scratch(int n, int n_rows, int H, int d, int dv) { return (long)(n / LC_CHUNK + n_rows) * H * d * (dv + 1); }

KA_API int ka_gated_chunks_bf16(const void* q, const void* k, const void* v, long stride, const float* pre, float tau, float q_scale,
                                float* state, long state_stride, const int* cu_q, const int* row_slot, float* raw, float* scratch, int n,
                                int n_rows, int H, int d, int dv, hipStream_t stream) {
    const char* who = "ka_gated_chunks_bf16";
    KA_CHECK(n >= 0 && n_rows >= 0 && H > 0 && ka_gated_chunks_supported(d, dv), "%s: heads of %d x %d not covered", who, d, dv);
    KA_CHECK(tau > 0.f && pre != nullptr, "%s: a decay needs its pre-activations and a positive tau", who);
    KA_CHECK((uintptr_t)q % 16 == 0 && (uintptr_t)k % 16 == 0 && (uintptr_t)v % 16 == 0 && stride % 8 == 0 && (uintptr_t)raw % 16 == 0 &&
             (uintptr_t)scratch % 16 == 0 && (uintptr_t)state % 16 == 0 && state_stride % 4 == 0, "%s: operands must be 16-byte aligned", who);
    KA_CHECK(state_stride >= (long)H * d * dv && stride >= (long)H * d && stride >= (long)H * dv, "%s: rows are shorter than their heads", who);
    const long n_chunks = n / LC_CHUNK + n_rows;
    KA_CHECK(H <= 65535 && n_rows <= 65535 && n_chunks <= 65535 && scratch != nullptr, "%s: too many heads, rows or chunks", who);
    if (n == 0 || n_rows == 0) return 0;
    GatedChunkArgs a;
    static_cast<LinearChunkArgs&>(a) = LinearChunkArgs{(const bf16_t*)q, (const bf16_t*)k, (const bf16_t*)v, stride, nullptr, state, state_stride,
                                                       cu_q, row_slot, raw, scratch, n_rows, H, d, dv, KA_ACT_NONE};
    a.pre = pre;
    a.factors = scratch + n_chunks * H * d * dv;
    a.per_tau = 1.f / tau;
    a.q_scale = q_scale;
    const int slices = ka_cdiv(dv, LC_SLICE), d32 = (d + 31) / 32 * 32, d64 = (d + 63) / 64 * 64;
    const size_t local_lds = sizeof(bf16_t) * (size_t)(2 * d32 + LC_SLICE) * LC_ROW + sizeof(float) * LC_BLOCKS * d64;
    const size_t read_lds = sizeof(bf16_t) * ((size_t)2 * LC_CHUNK * (d32 + LC_PAD) + (size_t)3 * LC_CHUNK * LC_ROW) +
                            sizeof(float) * ((size_t)LC_CHUNK * (d32 + 4) + (size_t)LC_BLOCKS * d32);
    static bool sized = false;
    if (!sized) {
        (void)hipFuncSetAttribute((const void*)gated_chunk_local_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
        (void)hipFuncSetAttribute((const void*)gated_chunk_read_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
        sized = true;
    }
    // (scores are shared by the slices a workgroup takes: all of them where heads and chunks fill the GPU)
    const int at_once = (long)H * n_chunks >= 2L * ka_compute_units() ? 1 : slices;
    hipLaunchKernelGGL(gated_chunk_local_kernel, dim3(H, n_chunks, slices), dim3(LC_THREADS), local_lds, stream, a);
    hipLaunchKernelGGL(linear_chunk_scan_kernel<true>, dim3(H, n_rows, ka_cdiv((long)d * dv, 4 * LC_THREADS)), dim3(LC_THREADS), 0, stream, a, a.factors);
    hipLaunchKernelGGL(gated_chunk_read_kernel, dim3(H, n_chunks, at_once), dim3(LC_THREADS), read_lds, stream, a);
    KA_LAUNCH_CHECK();
    return 0;
}
