// The linears of routed experts on the matrix cores (bf16): the pairs (token, choice) of a step come listed by expert, in
// runs that start on multiples of 128 rows of the list (ka_experts_sort), and a workgroup multiplies one tile of 128 list
// rows by 256 rows of its expert's weights (ka_listed_tiles.h): out[row] = act(a[row'] W_e^T).
//
//  * the first linear gathers: list row i holds pair p = sorted[i] (-1: an unused row), whose input is row p / gather_div
//    of `a`; its output goes to row i of `out` (the hidden rows stay in list order);
//  * the second linear scatters: its input is row i of `a`, its output goes to row p of `out`;
//  * gated (KA_ACT_GATED): weight rows 2j and 2j + 1 are gate and value of output j, as in every gated linear here, with or
//    without clamps (KaGateClamp).
//
// The weights are the row operand: a lane ends with outputs of ONE list row, four neighbours at a time, so the pair of a
// gated output meets in a lane's registers.
#include "ka_common.h"
#include "ka_listed_tiles.h"

typedef __attribute__((ext_vector_type(2))) __bf16 eb_bf16x2;

template <bool TAIL>
__global__ void __launch_bounds__(256)
experts_gemm_kernel(const bf16_t* __restrict__ a, long lda, int gather_div, const bf16_t* __restrict__ W, const int* __restrict__ sorted,
                    const int* __restrict__ tile_expert, int N, int K, int act, KaGateClamp clamp, void* __restrict__ out, long ldo,
                    int scatter, int out_f32) {
    extern __shared__ __attribute__((aligned(16))) bf16_t eb_lds[];
    const int tile = blockIdx.y;
    const int e = tile_expert[tile];
    if (e < 0) return;                                   // (the unused end of the list: the whole workgroup)
    const int wave = threadIdx.x / KA_WAVE, lane = threadIdx.x % KA_WAVE;
    const int col = lane % 32, half = lane / 32;
    const int o0 = blockIdx.x * KL_COLS + wave * 64;
    const int i0 = tile * KL_ROWS;
    int pr[4];
#pragma unroll
    for (int rb = 0; rb < 4; ++rb) pr[rb] = sorted[i0 + rb * 32 + col];
    // rows past the end, and unused rows of the list, are clamped for the loads and not stored
    auto list_row = [&](int r) { return a + (gather_div > 0 ? (long)max(sorted[i0 + r], 0) / gather_div : (long)i0 + r) * lda; };
    auto weight_row = [&](int r) { return W + ((size_t)e * N + min((int)blockIdx.x * KL_COLS + r, N - 1)) * K; };
    kl_floatx16 acc[2][4];
    const bool swap[2] = {false, false};
    kl_tile_product<TAIL, false>(eb_lds, K, o0 < N, swap, list_row, weight_row, acc);
    if (o0 >= N) return;
    const bool gated = ka_act_gated(act);
#pragma unroll
    for (int rb = 0; rb < 4; ++rb) {
        const int p = pr[rb];
        if (p < 0) continue;
        const long row = scatter ? (long)p : (long)i0 + rb * 32 + col;
#pragma unroll
        for (int wb = 0; wb < 2; ++wb) {
            const kl_floatx16& acc_here = acc[wb][rb];
            // register i: weight row o0 + 32 wb + (i / 4) * 8 + half * 4 + i % 4 of the lane's list row
#pragma unroll
            for (int g4 = 0; g4 < 4; ++g4) {
                const int o = o0 + wb * 32 + g4 * 8 + half * 4;
                if (gated) {
                    if (o + 3 < N) {
                        eb_bf16x2 y;
                        y[0] = (bf16_t)ka_gate_product<true>(act, clamp, acc_here[g4 * 4], acc_here[g4 * 4 + 1]);
                        y[1] = (bf16_t)ka_gate_product<true>(act, clamp, acc_here[g4 * 4 + 2], acc_here[g4 * 4 + 3]);
                        *reinterpret_cast<eb_bf16x2*>(reinterpret_cast<bf16_t*>(out) + row * ldo + o / 2) = y;
                    } else if (o + 1 < N) {
                        reinterpret_cast<bf16_t*>(out)[row * ldo + o / 2] = (bf16_t)ka_gate_product<true>(act, clamp, acc_here[g4 * 4], acc_here[g4 * 4 + 1]);
                    }
                } else if (out_f32) {
                    float* op = reinterpret_cast<float*>(out) + row * ldo + o;
                    if (o + 3 < N) {
                        *reinterpret_cast<float4*>(op) = make_float4(acc_here[g4 * 4], acc_here[g4 * 4 + 1], acc_here[g4 * 4 + 2], acc_here[g4 * 4 + 3]);
                    } else {
#pragma unroll
                        for (int x = 0; x < 4; ++x)
                            if (o + x < N) op[x] = acc_here[g4 * 4 + x];
                    }
                } else {
                    bf16_t* op = reinterpret_cast<bf16_t*>(out) + row * ldo + o;
                    kl_bf16x4 y;
#pragma unroll
                    for (int x = 0; x < 4; ++x) y[x] = (bf16_t)(ka_act_base(act) ? ka_activate_fast(act, acc_here[g4 * 4 + x]) : acc_here[g4 * 4 + x]);
                    if (o + 3 < N && ldo % 4 == 0) {
                        *reinterpret_cast<kl_bf16x4*>(op) = y;
                    } else {
#pragma unroll
                        for (int x = 0; x < 4; ++x)
                            if (o + x < N) op[x] = y[x];
                    }
                }
            }
        }
    }
}

KA_API int ka_experts_gemm_tile() { return KL_ROWS; }

// Whether the kernel covers these sizes and this alignment.
KA_API int ka_experts_gemm_supported(long lda, int N, int K, long ldo, int act, int out_f32) {
    const int n_out = ka_act_outputs(act, N);
    return K > 0 && K % 16 == 0 && lda % 8 == 0 && N > 0 && (!ka_act_gated(act) || (N % 4 == 0 && ldo % 2 == 0 && !out_f32)) &&
           (!out_f32 || ldo % 4 == 0) && ldo >= n_out ? 1 : 0;
}

KA_API int ka_experts_gemm_bf16(const void* a, long lda, int gather_div, const void* W, const int* sorted, const int* tile_expert,
                                int n_tiles, int N, int K, int act, int clamped, float limit, float slope, float shift, void* out,
                                long ldo, int scatter, int out_f32, hipStream_t stream) {
    const char* who = "ka_experts_gemm_bf16";
    KA_CHECK(!clamped || ka_act_gated(act), "%s: clamps are a gated linear's", who);
    const KaGateClamp clamp{clamped, limit, slope, shift};
    KA_CHECK(n_tiles >= 0 && n_tiles <= 65535 && gather_div >= 0, "%s: bad sizes (%d tiles)", who, n_tiles);
    KA_CHECK(ka_act_known(act) && ka_experts_gemm_supported(lda, N, K, ldo, act, out_f32), "%s: sizes N=%d K=%d not covered", who, N, K);
    KA_CHECK((uintptr_t)a % 16 == 0 && (uintptr_t)W % 16 == 0 && (uintptr_t)out % 16 == 0, "%s: operands must be 16-byte aligned", who);
    if (n_tiles == 0) return 0;
    const dim3 grid((N + KL_COLS - 1) / KL_COLS, n_tiles);
    static bool sized = false;
    if (!sized) {
        (void)hipFuncSetAttribute((const void*)experts_gemm_kernel<false>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
        (void)hipFuncSetAttribute((const void*)experts_gemm_kernel<true>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
        sized = true;
    }
    if (K % KL_SLAB == 0)
        hipLaunchKernelGGL(experts_gemm_kernel<false>, grid, dim3(256), KL_LDS_BYTES, stream, (const bf16_t*)a, lda, gather_div, (const bf16_t*)W,
                           sorted, tile_expert, N, K, act, clamp, out, ldo, scatter, out_f32);
    else
        hipLaunchKernelGGL(experts_gemm_kernel<true>, grid, dim3(256), KL_LDS_BYTES, stream, (const bf16_t*)a, lda, gather_div, (const bf16_t*)W,
                           sorted, tile_expert, N, K, act, clamp, out, ldo, scatter, out_f32);
    KA_LAUNCH_CHECK();
    return 0;
}

// ----------------------------------------------------------------------------
// The same linears for a step of few pairs (a decode step), where all that matters is to read every chosen expert's
// weights once: no lists are made beforehand, and weights go from memory to the matrix cores without LDS. A workgroup owns
// 16 weight rows of one expert; it looks through the choices for its expert's pairs (an expert that nobody chose ends there), its
// four waves take every fourth step of 64 inputs each and their sums meet in LDS. Weights are the row operand and pairs
// the columns, 16 or 32 at a time: a lane ends with four neighbouring outputs of one pair.
// ----------------------------------------------------------------------------
constexpr int EF_ROWS = 16;
constexpr int EF_MAX_PAIRS = 512;
constexpr int EF_WAVES = 4;
typedef __attribute__((ext_vector_type(8))) __bf16 ef_bf16x8;
typedef __attribute__((ext_vector_type(4))) float ef_floatx4;

struct ExpertsFewArgs {
    const bf16_t* a;
    long lda;
    int gather_div;             // the input of pair p is row p / gather_div of `a`
    const bf16_t* W;            // [E, N, K]
    const int* chosen;
    int n_pairs, N, K, act;
    KaGateClamp clamp;
    void* out;                  // row p: the outputs of pair p
    long ldo;
    int out_f32;
};

template <int MB, int U>
__device__ __forceinline__ void ef_columns(const ExpertsFewArgs& g, const bf16_t* W, const int* list, int count, int first, int row0,
                                           float* sums) {
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / KA_WAVE), lane = threadIdx.x % KA_WAVE;
    const int col = lane % 16, quarter = lane / 16;
    const bf16_t* w = W + (size_t)min(row0 + col, g.N - 1) * g.K;          // (rows past the end: not stored)
    const bf16_t* x[MB];
    int pair[MB];
#pragma unroll
    for (int m = 0; m < MB; ++m) {
        pair[m] = list[min(first + m * 16 + col, count - 1)];              // (columns past the last pair repeat it: not stored)
        x[m] = g.a + (size_t)(pair[m] / g.gather_div) * g.lda;
    }
    ef_floatx4 acc[MB];
#pragma unroll
    for (int m = 0; m < MB; ++m) acc[m] = ef_floatx4{0.f, 0.f, 0.f, 0.f};
    // (two products a step of 64 inputs: a lane's 16 are neighbours, a row's 64 a whole line; which of them meet in which
    // product is the same for weights and pairs)
    for (int k0 = wave * 64 + quarter * 16; k0 - quarter * 16 < g.K; k0 += EF_WAVES * 32 * U) {
        ef_bf16x8 wv[U], xv[U][MB];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int k = k0 + u / 2 * EF_WAVES * 64 + u % 2 * 8;
            const bool in = k < g.K;
#pragma unroll
            for (int i = 0; i < 8; ++i) wv[u][i] = (bf16_t)0.f;
            if (in) wv[u] = __builtin_nontemporal_load(reinterpret_cast<const ef_bf16x8*>(w + k));
#pragma unroll
            for (int m = 0; m < MB; ++m) {
#pragma unroll
                for (int i = 0; i < 8; ++i) xv[u][m][i] = (bf16_t)0.f;
                if (in) xv[u][m] = *reinterpret_cast<const ef_bf16x8*>(x[m] + k);
            }
        }
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
            for (int m = 0; m < MB; ++m) acc[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv[u], xv[u][m], acc[m], 0, 0, 0);
    }
#pragma unroll
    for (int m = 0; m < MB; ++m) *reinterpret_cast<ef_floatx4*>(sums + ((wave * MB + m) * KA_WAVE + lane) * 4) = acc[m];
    __syncthreads();
    if (wave >= MB) return;
    ef_floatx4 y = ef_floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int v = 0; v < EF_WAVES; ++v) y += *reinterpret_cast<const ef_floatx4*>(sums + ((v * MB + wave) * KA_WAVE + lane) * 4);
    if (first + wave * 16 + col >= count) return;
    const size_t row = (size_t)pair[MB == 1 ? 0 : wave] * g.ldo;
    const int o = row0 + quarter * 4;
    if (ka_act_gated(g.act)) {
        bf16_t* op = reinterpret_cast<bf16_t*>(g.out) + row + o / 2;
        if (o + 1 < g.N) op[0] = (bf16_t)ka_gate_product<true>(g.act, g.clamp, y[0], y[1]);
        if (o + 3 < g.N) op[1] = (bf16_t)ka_gate_product<true>(g.act, g.clamp, y[2], y[3]);
        return;
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        if (o + r >= g.N) continue;
        const float v = ka_activate_fast(g.act, y[r]);
        if (g.out_f32) reinterpret_cast<float*>(g.out)[row + o + r] = v;
        else reinterpret_cast<bf16_t*>(g.out)[row + o + r] = (bf16_t)v;
    }
}

__global__ void __launch_bounds__(EF_WAVES * KA_WAVE) experts_few_kernel(ExpertsFewArgs g) {
    __shared__ int list[EF_MAX_PAIRS];
    __shared__ __attribute__((aligned(16))) float sums[EF_WAVES * 2 * KA_WAVE * 4];
    const int e = blockIdx.y, lane = threadIdx.x % KA_WAVE;
    // (every wave makes the list by itself: all write the same numbers)
    int mine[EF_MAX_PAIRS / KA_WAVE];
#pragma unroll
    for (int i = 0; i < EF_MAX_PAIRS / KA_WAVE; ++i) mine[i] = i * KA_WAVE + lane < g.n_pairs ? g.chosen[i * KA_WAVE + lane] : -1;
    int count = 0;
#pragma unroll
    for (int i = 0; i < EF_MAX_PAIRS / KA_WAVE; ++i) {
        const unsigned long long hit = __builtin_amdgcn_ballot_w64(mine[i] == e);
        if (mine[i] == e) list[count + __popcll(hit & ((1ull << lane) - 1))] = i * KA_WAVE + lane;
        count += __popcll(hit);
    }
    if (count == 0) return;
    __syncthreads();
    const bf16_t* W = g.W + (size_t)e * g.N * g.K;
    const int row0 = blockIdx.x * EF_ROWS;
    for (int first = 0; first < count;) {
        if (count - first <= 16) {
            ef_columns<1, 8>(g, W, list, count, first, row0, sums);
            first += 16;
        } else {
            ef_columns<2, 4>(g, W, list, count, first, row0, sums);
            first += 32;
        }
        __syncthreads();
    }
}

// Whether the kernel takes the call: inputs in steps of 8, 16-byte rows, gated pairs inside N.
KA_API int ka_experts_few_supported(int n_pairs, long lda, int N, int K, int act) {
    return n_pairs > 0 && n_pairs <= EF_MAX_PAIRS && N > 0 && K > 0 && K % 8 == 0 && lda % 8 == 0 && (!ka_act_gated(act) || N % 2 == 0) ? 1 : 0;
}

KA_API int ka_experts_few_bf16(const void* a, long lda, int gather_div, const void* W, const int* chosen, int n_pairs, int E, int N, int K,
                               int act, int clamped, float limit, float slope, float shift, void* out, long ldo, int out_f32,
                               hipStream_t stream) {
    const char* who = "ka_experts_few_bf16";
    KA_CHECK(!clamped || ka_act_gated(act), "%s: clamps are a gated linear's", who);
    KA_CHECK(ka_act_known(act) && ka_experts_few_supported(n_pairs, lda, N, K, act), "%s: %d pairs, N=%d K=%d not covered", who, n_pairs, N, K);
    KA_CHECK(E > 0 && E <= 65535 && gather_div > 0 && lda >= K && ldo >= (ka_act_gated(act) ? N / 2 : N), "%s: bad sizes", who);
    KA_CHECK(!ka_act_gated(act) || !out_f32, "%s: a gated linear writes bf16", who);
    KA_CHECK((uintptr_t)a % 16 == 0 && (uintptr_t)W % 16 == 0, "%s: operands must be 16-byte aligned", who);
    const ExpertsFewArgs g{(const bf16_t*)a, lda, gather_div, (const bf16_t*)W, chosen, n_pairs, N, K, act, {clamped, limit, slope, shift}, out, ldo, out_f32};
    hipLaunchKernelGGL(experts_few_kernel, dim3(ka_cdiv(N, EF_ROWS), E), dim3(EF_WAVES * KA_WAVE), 0, stream, g);
    KA_LAUNCH_CHECK();
    return 0;
}
