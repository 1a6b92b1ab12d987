// Latent attention over long portions of prompts (bf16): the cached latents that a portion's queries see are lifted to keys
// and values per head, k = W_uk c and v = W_uv c, into pages laid out as the attention kernels read them (keys [pages, H, 16,
// d], values [pages, H, dv, 16]), so that a score costs d multiply-adds instead of the latent's size, and so does not every
// query's every head. The lifted pages are scratch of the step; the cache holds latents as before.
//
// Which rows of a step are lifted is decided on the device, from what the step holds, so that a captured step can be
// replayed on others of its size: those that bring at least `from` tokens. The rest of the step (decoded tokens, short
// portions) goes the other way, queries against latents, through the kernels that know how to pass over rows
// (attn_biased_kernel's range of tokens a row, heads_linear_kernel's `skip`).
#include "ka_common.h"
#include "ka_listed_tiles.h"

constexpr int LE_PAGE = 16;
constexpr int LE_MAX_ROWS = 1024;

// ----------------------------------------------------------------------------
// What is to be lifted, one workgroup. Row r brings cu_q[r + 1] - cu_q[r] tokens; if at least `from`, and it has keys, the pages
// from the one its first token's window starts in (kv_lo) to its last key's are lifted, side by side from lifted page
// base_r on: list[p * 16 + o] = the place in the cache of the key whose lifted place that is (-1: a page that was given
// back, and the places behind the last one up to the end of its tile), table[r][logical page] = lifted page (the neighbours
// of a row's first and last one, which a kernel may look up and then mask, -1), used[0] = lifted places in all, lifted[t] = 1
// for every token of a row that brings at least `from`, else 0. The caller's `capacity` holds every such row's pages (rows that would
// not fit are given none, never a place outside).
// ----------------------------------------------------------------------------
__global__ void __launch_bounds__(1024)
latent_expand_plan_kernel(const int* __restrict__ cu_q, const int* __restrict__ kv_len, const int* __restrict__ kv_lo,
                          const int* __restrict__ token_row, const int* __restrict__ block_table, int max_pages, int n, int n_rows, int from,
                          int capacity, int* __restrict__ list, int* __restrict__ table, int* __restrict__ used, int* __restrict__ lifted) {
    __shared__ int first_s[LE_MAX_ROWS], base_s[LE_MAX_ROWS + 1], wave_s[16];
    const int tid = threadIdx.x, lane = tid % KA_WAVE, wave = tid / KA_WAVE;
    int count = 0;
    if (tid < n_rows) {
        const int t0 = cu_q[tid], q = cu_q[tid + 1] - t0, keys = kv_len[tid];
        if (q >= from && keys > 0) {
            const int first = min(kv_lo ? kv_lo[t0] : 0, keys - 1) / LE_PAGE;
            first_s[tid] = first;
            count = min((keys - 1) / LE_PAGE, max_pages - 1) - first + 1;
        }
    }
    // running sums over the rows (counts of pages: exact in fp32)
    const int upto = (int)ka_wave_running_sum((float)count);
    if (lane == KA_WAVE - 1) wave_s[wave] = upto;
    __syncthreads();
    int before = 0;
    for (int w = 0; w < wave; ++w) before += wave_s[w];
    // (rows behind the one that would not fit are not lifted either)
    if (tid < n_rows) base_s[tid + 1] = before + upto;
    if (tid == 0) base_s[0] = 0;
    __syncthreads();
    int lo = 0, hi = n_rows;                    // the most rows whose pages fit
    while (lo < hi) {
        const int mid = (lo + hi + 1) / 2;
        if (base_s[mid] <= capacity) lo = mid; else hi = mid - 1;
    }
    const int rows = lo, total = base_s[rows];
    if (tid == 0) used[0] = total * LE_PAGE;
    for (int i = tid; i < total; i += blockDim.x) {
        int a = 0, b = rows - 1;                // the row whose pages hold lifted page i: the last that starts at or before it
        while (a < b) {
            const int mid = (a + b + 1) / 2;
            if (base_s[mid] <= i) a = mid; else b = mid - 1;
        }
        const int logical = first_s[a] + (i - base_s[a]);
        const int page = block_table[(size_t)a * max_pages + logical];
        table[(size_t)a * max_pages + logical] = i;
        if (i == base_s[a] && logical > 0) table[(size_t)a * max_pages + logical - 1] = -1;
        if (i + 1 == base_s[a + 1] && logical + 1 < max_pages) table[(size_t)a * max_pages + logical + 1] = -1;
        for (int o = 0; o < LE_PAGE; ++o) list[(size_t)i * LE_PAGE + o] = page < 0 ? -1 : page * LE_PAGE + o;
    }
    const int end = min((total * LE_PAGE + KL_ROWS - 1) / KL_ROWS * KL_ROWS, capacity * LE_PAGE);
    for (int i = total * LE_PAGE + tid; i < end; i += blockDim.x) list[i] = -1;
    for (int t = tid; t < n; t += blockDim.x) {
        const int r = token_row[t];
        lifted[t] = cu_q[r + 1] - cu_q[r] >= from ? 1 : 0;
    }
}

// ----------------------------------------------------------------------------
// The lift itself: 128 listed places by 256 rows of [W_uk; W_uv] a workgroup. Keys: a lane holds four neighbouring channels of
// one place (weights as the row operand); values: four neighbouring places of one channel (list rows as the row operand).
// Either leaves as 8-byte pieces of its page.
// ----------------------------------------------------------------------------
template <bool TAIL>
__global__ void __launch_bounds__(256)
latent_expand_kernel(const bf16_t* __restrict__ cache, long row_dim, const bf16_t* __restrict__ W, const int* __restrict__ list,
                     const int* __restrict__ used, int H, int d, int dv, int K, bf16_t* __restrict__ keys, bf16_t* __restrict__ values) {
    extern __shared__ __attribute__((aligned(16))) bf16_t le_lds[];
    const int i0 = blockIdx.y * KL_ROWS;
    if (i0 >= used[0]) return;                           // (the whole workgroup)
    const int wave = threadIdx.x / KA_WAVE, lane = threadIdx.x % KA_WAVE;
    const int col = lane % 32, half = lane / 32;
    const int n_keys = H * d, N = n_keys + H * dv;
    const int o0 = blockIdx.x * KL_COLS + wave * 64;
    auto list_row = [&](int r) { return cache + (long)max(list[i0 + r], 0) * row_dim; };
    auto weight_row = [&](int r) { return W + (size_t)min((int)blockIdx.x * KL_COLS + r, N - 1) * K; };
    kl_floatx16 acc[2][4];
    const bool swap[2] = {o0 >= n_keys, o0 + 32 >= n_keys};     // (n_keys is a multiple of 32: a block of 32 is all keys or all values)
    kl_tile_product<TAIL, true>(le_lds, K, o0 < N, swap, list_row, weight_row, acc);
#pragma unroll
    for (int wb = 0; wb < 2; ++wb) {
        const int ob = o0 + wb * 32;
        if (ob >= N) continue;
#pragma unroll
        for (int rb = 0; rb < 4; ++rb) {
#pragma unroll
            for (int g4 = 0; g4 < 4; ++g4) {
                kl_bf16x4 y;
#pragma unroll
                for (int x = 0; x < 4; ++x) y[x] = (bf16_t)acc[wb][rb][g4 * 4 + x];
                if (!swap[wb]) {
                    const int i = i0 + rb * 32 + col, o = ob + g4 * 8 + half * 4;
                    const int head = o / d, ch = o % d;                    // (d is a multiple of 4)
                    if (i < used[0])
                        *reinterpret_cast<kl_bf16x4*>(keys + (((size_t)(i / LE_PAGE) * H + head) * LE_PAGE + i % LE_PAGE) * d + ch) = y;
                } else {
                    const int i = i0 + rb * 32 + g4 * 8 + half * 4, o = ob + col - n_keys;
                    const int head = o / dv, ch = o % dv;
                    if (i < used[0] && o < H * dv)                          // (places in use are whole pages)
                        *reinterpret_cast<kl_bf16x4*>(values + (((size_t)(i / LE_PAGE) * H + head) * dv + ch) * LE_PAGE + i % LE_PAGE) = y;
                }
            }
        }
    }
}

// Whether the lift covers these sizes: keys of all heads in whole blocks of 32 weight rows, latents in steps of 16.
KA_API int ka_latent_expand_supported(int H, int d, int dv, int rank, long row_dim) {
    return H > 0 && d > 0 && d % 4 == 0 && (H * d) % 32 == 0 && dv > 0 && rank > 0 && rank % 16 == 0 && row_dim >= rank && row_dim % 8 == 0 ? 1 : 0;
}

KA_API int ka_latent_expand_max_rows() { return LE_MAX_ROWS; }

// capacity: lifted pages there is room for, a multiple of 8 (list: capacity * 16 numbers; table: [n_rows, max_pages]; lifted: n).
KA_API int ka_latent_expand_plan(const int* cu_q, const int* kv_len, const int* kv_lo, const int* token_row, const int* block_table,
                                 int max_pages, int n, int n_rows, int from, int capacity, int* list, int* table, int* used, int* lifted,
                                 hipStream_t stream) {
    const char* who = "ka_latent_expand_plan";
    KA_CHECK(n >= 0 && n_rows >= 0 && n_rows <= LE_MAX_ROWS && from > 0 && max_pages > 0, "%s: bad sizes", who);
    KA_CHECK(capacity > 0 && capacity % (KL_ROWS / LE_PAGE) == 0 && capacity < (1 << 23), "%s: room for %d pages", who, capacity);
    if (n == 0) return 0;
    hipLaunchKernelGGL(latent_expand_plan_kernel, dim3(1), dim3(1024), 0, stream, cu_q, kv_len, kv_lo, token_row, block_table, max_pages, n,
                       n_rows, from, capacity, list, table, used, lifted);
    KA_LAUNCH_CHECK();
    return 0;
}

KA_API int ka_latent_expand_bf16(const void* cache, long row_dim, const void* W, const int* list, const int* used, int capacity, int H,
                                 int d, int dv, int rank, void* keys, void* values, hipStream_t stream) {
    const char* who = "ka_latent_expand_bf16";
    KA_CHECK(ka_latent_expand_supported(H, d, dv, rank, row_dim), "%s: %d heads of %d / %d channels over %d not covered", who, H, d, dv, rank);
    KA_CHECK(capacity > 0 && capacity % (KL_ROWS / LE_PAGE) == 0 && capacity / (KL_ROWS / LE_PAGE) <= 65535, "%s: room for %d pages", who, capacity);
    KA_CHECK((uintptr_t)cache % 16 == 0 && (uintptr_t)W % 16 == 0 && (uintptr_t)keys % 16 == 0 && (uintptr_t)values % 16 == 0,
             "%s: operands must be 16-byte aligned", who);
    const int N = H * (d + dv);
    const dim3 grid((N + KL_COLS - 1) / KL_COLS, capacity / (KL_ROWS / LE_PAGE));
    static bool sized = false;
    if (!sized) {
        (void)hipFuncSetAttribute((const void*)latent_expand_kernel<false>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
        (void)hipFuncSetAttribute((const void*)latent_expand_kernel<true>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
        sized = true;
    }
    if (rank % KL_SLAB == 0)
        hipLaunchKernelGGL(latent_expand_kernel<false>, grid, dim3(256), KL_LDS_BYTES, stream, (const bf16_t*)cache, row_dim, (const bf16_t*)W, list,
                           used, H, d, dv, rank, (bf16_t*)keys, (bf16_t*)values);
    else
        hipLaunchKernelGGL(latent_expand_kernel<true>, grid, dim3(256), KL_LDS_BYTES, stream, (const bf16_t*)cache, row_dim, (const bf16_t*)W, list,
                           used, H, d, dv, rank, (bf16_t*)keys, (bf16_t*)values);
    KA_LAUNCH_CHECK();
    return 0;
}
