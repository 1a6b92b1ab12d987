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
