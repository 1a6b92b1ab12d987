// Kernels of attention without a softmax, run as a recurrence: the walk over a row's tokens one by one, and the norm of
// what it reads. fp32 or bf16 storage of what the projections made; activations, decays, the state and all sums are fp32.
#include "ka_common.h"
#include "ka_decay.h"

constexpr int LA_THREADS = 256;

// ----------------------------------------------------------------------------
// Per request and head a state S [dv, d] (value channel by key channel), fp32. For every token of a row, in order,
//     S <- decay_h S + v k^T,    o = S q,         q, k, v = act(projected)
// and o [dv] is left in `raw` in fp32. A value channel's row of S is independent of the others: a head is dealt out over
// workgroups by slices of value channels (blockIdx.z) and over groups of LI lanes, a lane holding four key channels (NV
// times) of NJ value channels in registers; a read-out is a sum over the LI lanes of a group inside the vector unit.
// Nothing passes between waves. One launch takes whatever a step holds: a prompt, a portion, single tokens. The next
// token's numbers are asked for before the current token's sums. A row without a request (slot < 0) gets zeros.
//
// GATED: instead of one decay per head, a decay per key channel computed from the token, a_i = sigmoid(pre_i)^(1 / tau) with
// fp32 pre [n, H d] (ka_decay.h), and queries times q_scale.
// ----------------------------------------------------------------------------
struct LinearAttentionArgs {
    const void* q;
    const void* k;
    const void* v;
    long stride;            // of the rows of q, k and v
    const float* decay;     // [H]
    float* state;           // [slots, state_stride]: S [H, dv, d]
    long state_stride;
    const int* cu_q;
    const int* row_slot;
    float* raw;             // [n, H dv]
    int H, d, dv, act, vectors;
    const float* pre;       // GATED: [n, H d]
    float per_tau, q_scale; // GATED: 1 / tau
};

template <typename T>
__device__ __forceinline__ float4 la_four(const T* p, int c, int d, bool vectors) {
    typedef __attribute__((ext_vector_type(4))) T vec;
    if (vectors) {
        if (c >= d) return make_float4(0.f, 0.f, 0.f, 0.f);
        const vec x = *reinterpret_cast<const vec*>(p + c);
        return make_float4(ka_to_float(x[0]), ka_to_float(x[1]), ka_to_float(x[2]), ka_to_float(x[3]));
    }
    return make_float4(c < d ? ka_to_float(p[c]) : 0.f, c + 1 < d ? ka_to_float(p[c + 1]) : 0.f, c + 2 < d ? ka_to_float(p[c + 2]) : 0.f,
                       c + 3 < d ? ka_to_float(p[c + 3]) : 0.f);
}

// (every activation of the table maps 0 to 0: channels behind the last stay out of the sums)
template <typename T>
__device__ __forceinline__ float la_act(int act, float x) {
    return sizeof(T) == 2 ? ka_activate_fast(act, x) : ka_activate(act, x);
}
template <typename T>
__device__ __forceinline__ float4 la_act4(int act, float4 x) {
    return make_float4(la_act<T>(act, x.x), la_act<T>(act, x.y), la_act<T>(act, x.z), la_act<T>(act, x.w));
}

template <typename T, int LI, int NV, int NJ, bool GATED>
__global__ void __launch_bounds__(LA_THREADS) linear_attention_kernel(LinearAttentionArgs a) {
    constexpr int JW = LA_THREADS / LI;
    const int head = blockIdx.x, row = blockIdx.y, tid = threadIdx.x;
    const int li = tid % LI, jr = tid / LI;
    const int d = a.d, dv = a.dv;
    const int j0 = blockIdx.z * (JW * NJ);
    const int t0 = a.cu_q[row], t1 = a.cu_q[row + 1];
    if (t0 >= t1) return;
    const int slot = a.row_slot[row];
    const size_t out_at = (size_t)head * dv, out_row = (size_t)a.H * dv;
    if (slot < 0) {
        for (int t = t0; t < t1; ++t)
#pragma unroll
            for (int m = 0; m < NJ; ++m) {
                const int j = j0 + m * JW + jr;
                if (li == 0 && j < dv) a.raw[(size_t)t * out_row + out_at + j] = 0.f;
            }
        return;
    }
    const bool vectors = a.vectors != 0;
    float* S_mem = a.state + (size_t)slot * a.state_stride + (size_t)head * dv * d;
    const T* qp = reinterpret_cast<const T*>(a.q) + (size_t)head * d;
    const T* kp = reinterpret_cast<const T*>(a.k) + (size_t)head * d;
    const T* vp = reinterpret_cast<const T*>(a.v) + (size_t)head * dv;
    const float keep = GATED ? 1.f : a.decay[head];
    float4 S[NJ][NV];
    int jc[NJ];             // (value channels behind the last are clamped for the loads and not stored)
#pragma unroll
    for (int m = 0; m < NJ; ++m) {
        const int j = j0 + m * JW + jr;
        jc[m] = min(j, dv - 1);
#pragma unroll
        for (int u = 0; u < NV; ++u) S[m][u] = la_four(S_mem + (size_t)jc[m] * d, (u * LI + li) * 4, d, d % 4 == 0);
    }
    float4 qn[NV], kn[NV], zn[GATED ? NV : 1];
    float vn[NJ];
    auto fetch = [&](int t) {
        const size_t at = (size_t)t * a.stride;
#pragma unroll
        for (int u = 0; u < NV; ++u) {
            qn[u] = la_four(qp + at, (u * LI + li) * 4, d, vectors);
            kn[u] = la_four(kp + at, (u * LI + li) * 4, d, vectors);
            if constexpr (GATED) zn[u] = la_four(a.pre + (size_t)t * a.H * d + (size_t)head * d, (u * LI + li) * 4, d, vectors);
        }
#pragma unroll
        for (int m = 0; m < NJ; ++m) vn[m] = ka_to_float(vp[at + jc[m]]);
    };
    fetch(t0);
    for (int t = t0; t < t1; ++t) {
        float4 q[NV], k[NV], w[GATED ? NV : 1];
        float v[NJ];
#pragma unroll
        for (int u = 0; u < NV; ++u) {
            q[u] = la_act4<T>(a.act, qn[u]);
            k[u] = la_act4<T>(a.act, kn[u]);
            if constexpr (GATED) {
                q[u] = make_float4(q[u].x * a.q_scale, q[u].y * a.q_scale, q[u].z * a.q_scale, q[u].w * a.q_scale);
                w[u] = make_float4(ka_decay<sizeof(T) == 2>(zn[u].x, a.per_tau), ka_decay<sizeof(T) == 2>(zn[u].y, a.per_tau),
                                   ka_decay<sizeof(T) == 2>(zn[u].z, a.per_tau), ka_decay<sizeof(T) == 2>(zn[u].w, a.per_tau));
            }
        }
#pragma unroll
        for (int m = 0; m < NJ; ++m) v[m] = la_act<T>(a.act, vn[m]);
        if (t + 1 < t1) fetch(t + 1);
#pragma unroll
        for (int m = 0; m < NJ; ++m) {
            float acc = 0.f;
#pragma unroll
            for (int u = 0; u < NV; ++u) {
                float4& s = S[m][u];
                const float4 f = GATED ? w[GATED ? u : 0] : make_float4(keep, keep, keep, keep);
                s.x = fmaf(f.x, s.x, k[u].x * v[m]);
                s.y = fmaf(f.y, s.y, k[u].y * v[m]);
                s.z = fmaf(f.z, s.z, k[u].z * v[m]);
                s.w = fmaf(f.w, s.w, k[u].w * v[m]);
                acc = fmaf(q[u].x, s.x, acc);
                acc = fmaf(q[u].y, s.y, acc);
                acc = fmaf(q[u].z, s.z, acc);
                acc = fmaf(q[u].w, s.w, acc);
            }
            acc = ka_lanes_reduce<1, LI>(acc, KaSum{});
            const int j = j0 + m * JW + jr;
            if (li == 0 && j < dv) a.raw[(size_t)t * out_row + out_at + j] = acc;
        }
    }
#pragma unroll
    for (int m = 0; m < NJ; ++m) {
        const int j = j0 + m * JW + jr;
        if (j >= dv) continue;
#pragma unroll
        for (int u = 0; u < NV; ++u) {
            const int c = (u * LI + li) * 4;
            float* p = S_mem + (size_t)j * d + c;
            if (d % 4 == 0) {
                if (c < d) *reinterpret_cast<float4*>(p) = S[m][u];
            } else {
                if (c < d) p[0] = S[m][u].x;
                if (c + 1 < d) p[1] = S[m][u].y;
                if (c + 2 < d) p[2] = S[m][u].z;
                if (c + 3 < d) p[3] = S[m][u].w;
            }
        }
    }
}

constexpr int LA_MAX_D = 512;

KA_API int ka_linear_attention_supported(int d, int dv) { return d > 0 && d <= LA_MAX_D && dv > 0 ? 1 : 0; }

template <bool GATED>
static int la_run(const char* who, const LinearAttentionArgs& given, int dtype, int n, int n_rows, hipStream_t stream);

KA_API int ka_linear_attention(const void* q, const void* k, const void* v, long stride, int dtype, const float* decay, float* state,
                               long state_stride, const int* cu_q, const int* row_slot, float* raw, int n, int n_rows, int H, int d,
                               int dv, int act, hipStream_t stream) {
    return la_run<false>("ka_linear_attention", {q, k, v, stride, decay, state, state_stride, cu_q, row_slot, raw, H, d, dv, act, 0, nullptr, 0.f, 1.f},
                         dtype, n, n_rows, stream);
}

// pre: fp32 [n, H d]; a key channel's decay is sigmoid(pre)^(1 / tau).
KA_API int ka_gated_linear_attention(const void* q, const void* k, const void* v, long stride, int dtype, const float* pre, float tau,
                                     float q_scale, float* state, long state_stride, const int* cu_q, const int* row_slot, float* raw,
                                     int n, int n_rows, int H, int d, int dv, hipStream_t stream) {
    const char* who = "ka_gated_linear_attention";
    KA_CHECK(tau > 0.f && pre != nullptr, "%s: a decay needs its pre-activations and a positive tau", who);
    return la_run<true>(who, {q, k, v, stride, nullptr, state, state_stride, cu_q, row_slot, raw, H, d, dv, KA_ACT_NONE, 0, pre, 1.f / tau, q_scale},
                        dtype, n, n_rows, stream);
}

template <bool GATED>
static int la_run(const char* who, const LinearAttentionArgs& given, int dtype, int n, int n_rows, hipStream_t stream) {
    const int H = given.H, d = given.d, dv = given.dv, act = given.act;
    const long stride = given.stride, state_stride = given.state_stride;
    const void *q = given.q, *k = given.k, *state = given.state;
    KA_CHECK(n >= 0 && n_rows >= 0 && H > 0 && ka_linear_attention_supported(d, dv), "%s: heads of %d x %d channels are not covered (keys up to %d)", who, d, dv, LA_MAX_D);
    KA_CHECK(dtype == KA_F32 || dtype == KA_BF16, "%s: unsupported dtype %d", who, dtype);
    KA_CHECK(ka_act_known(act) && !ka_act_gated(act), "%s: unknown activation %d", who, act);
    KA_CHECK(state_stride >= (long)H * d * dv && (uintptr_t)state % 16 == 0 && (d % 4 != 0 || state_stride % 4 == 0), "%s: the state rows are too short or not aligned", who);
    KA_CHECK(stride >= (long)H * d && stride >= (long)H * dv, "%s: rows are shorter than their heads", who);
    KA_CHECK(H <= 65535 && n_rows <= 65535, "%s: too many heads or rows", who);
    if (n == 0 || n_rows == 0) return 0;
    const size_t align = dtype == KA_F32 ? 16 : 8;
    const int vectors = d % 4 == 0 && stride % 4 == 0 && (uintptr_t)q % align == 0 && (uintptr_t)k % align == 0;
    LinearAttentionArgs a = given;
    a.vectors = vectors && (!GATED || (uintptr_t)given.pre % 16 == 0);
    const int lanes = d <= 32 ? 8 : d <= 64 ? 16 : d <= 128 ? 32 : 64;
    // (few workgroups: a value channel a group of lanes; many: four, so that a token's keys and queries serve four)
    const int jw = LA_THREADS / lanes;
    const int nj = (long)H * n_rows * ka_cdiv(dv, jw) >= 8L * ka_compute_units() ? 4 : 1;
    const dim3 grid(H, n_rows, ka_cdiv(dv, jw * nj));
#define LA_LAUNCH(T, LI, NV, NJ) hipLaunchKernelGGL((linear_attention_kernel<T, LI, NV, NJ, GATED>), grid, dim3(LA_THREADS), 0, stream, a)
#define LA_LAUNCH_NJ(T, LI, NV)          \
    if (nj == 4) LA_LAUNCH(T, LI, NV, 4); \
    else LA_LAUNCH(T, LI, NV, 1)
#define LA_LAUNCH_ALL(T)                                \
    if (lanes == 8) { LA_LAUNCH_NJ(T, 8, 1); }          \
    else if (lanes == 16) { LA_LAUNCH_NJ(T, 16, 1); }   \
    else if (lanes == 32) { LA_LAUNCH_NJ(T, 32, 1); }   \
    else if (d <= 256) { LA_LAUNCH_NJ(T, 64, 1); }      \
    else { LA_LAUNCH_NJ(T, 64, 2); }
    if (dtype == KA_F32) { LA_LAUNCH_ALL(float) } else { LA_LAUNCH_ALL(bf16_t) }
#undef LA_LAUNCH_ALL
#undef LA_LAUNCH_NJ
#undef LA_LAUNCH
    KA_LAUNCH_CHECK();
    return 0;
}

// ----------------------------------------------------------------------------
// out[t] = x[t] / sqrt(mean(x[t]^2) + eps) * gain * sigmoid(gate[t]) over whole fp32 rows x [n, dim] (gain, gate optional):
// a workgroup per row, which stays in registers where it has up to 4 PIECES LA_THREADS channels in pieces of four.
// ----------------------------------------------------------------------------
__device__ __forceinline__ float la_block_sum(float v, float* smem) {
    v = ka_wave_sum(v);
    if (threadIdx.x % KA_WAVE == 0) smem[threadIdx.x / KA_WAVE] = v;
    __syncthreads();
    float total = 0.f;
#pragma unroll
    for (int w = 0; w < LA_THREADS / KA_WAVE; ++w) total += smem[w];
    return total;
}

template <typename T>
__device__ __forceinline__ float la_sigmoid(float x) {
    return sizeof(T) == 2 ? __fdividef(1.0f, 1.0f + __expf(-x)) : 1.0f / (1.0f + expf(-x));
}

template <typename T, int PIECES>
__global__ void __launch_bounds__(LA_THREADS)
gated_rmsnorm_kernel(const float* __restrict__ x, const float* __restrict__ gain, const T* __restrict__ gate, long gate_stride,
                     T* __restrict__ out, int dim, float eps) {
    __shared__ float smem[LA_THREADS / KA_WAVE];
    typedef __attribute__((ext_vector_type(4))) T vec;
    const int t = blockIdx.x, tid = threadIdx.x;
    const float* row = x + (size_t)t * dim;
    const T* g = gate ? gate + (size_t)t * gate_stride : nullptr;
    T* o = out + (size_t)t * dim;
    if constexpr (PIECES > 0) {
        float4 v[PIECES];
        vec gt[PIECES];
        float s = 0.f;
#pragma unroll
        for (int p = 0; p < PIECES; ++p) {
            const int c = (p * LA_THREADS + tid) * 4;
            if (c < dim) {
                v[p] = *reinterpret_cast<const float4*>(row + c);
                if (g) gt[p] = *reinterpret_cast<const vec*>(g + c);
                s += v[p].x * v[p].x + v[p].y * v[p].y + v[p].z * v[p].z + v[p].w * v[p].w;
            }
        }
        const float r = 1.0f / sqrtf(la_block_sum(s, smem) / (float)dim + eps);
#pragma unroll
        for (int p = 0; p < PIECES; ++p) {
            const int c = (p * LA_THREADS + tid) * 4;
            if (c < dim) {
                float y[4] = {v[p].x * r, v[p].y * r, v[p].z * r, v[p].w * r};
                vec b;
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    if (gain) y[e] *= gain[c + e];
                    if (g) y[e] *= la_sigmoid<T>(ka_to_float(gt[p][e]));
                    b[e] = ka_from_float<T>(y[e]);
                }
                *reinterpret_cast<vec*>(o + c) = b;
            }
        }
    } else {
        float s = 0.f;
        for (int c = tid; c < dim; c += LA_THREADS) s += row[c] * row[c];
        const float r = 1.0f / sqrtf(la_block_sum(s, smem) / (float)dim + eps);
        for (int c = tid; c < dim; c += LA_THREADS) {
            float y = row[c] * r * (gain ? gain[c] : 1.f);
            if (g) y *= la_sigmoid<T>(ka_to_float(g[c]));
            o[c] = ka_from_float<T>(y);
        }
    }
}

KA_API int ka_gated_rmsnorm(const float* x, const float* gain, const void* gate, long gate_stride, void* out, int dtype, int n, int dim,
                            float eps, hipStream_t stream) {
    const char* who = "ka_gated_rmsnorm";
    KA_CHECK(n >= 0 && dim > 0 && eps >= 0.f && (gate == nullptr || gate_stride >= dim), "%s: bad sizes", who);
    KA_CHECK(dtype == KA_F32 || dtype == KA_BF16, "%s: unsupported dtype %d", who, dtype);
    if (n == 0) return 0;
    const size_t align = dtype == KA_F32 ? 16 : 8;
    const bool vectors = dim % 4 == 0 && (uintptr_t)x % 16 == 0 && (uintptr_t)out % align == 0 &&
                         (gate == nullptr || ((uintptr_t)gate % align == 0 && gate_stride % 4 == 0));
    const int need = ka_cdiv(dim, 4 * LA_THREADS);
    const int pieces = !vectors || need > 8 ? 0 : need <= 1 ? 1 : need <= 2 ? 2 : need <= 4 ? 4 : 8;
#define LA_NORM(T, P) \
    hipLaunchKernelGGL((gated_rmsnorm_kernel<T, P>), dim3(n), dim3(LA_THREADS), 0, stream, x, gain, (const T*)gate, gate_stride, (T*)out, dim, eps)
#define LA_NORM_ALL(T)                   \
    switch (pieces) {                    \
        case 1: LA_NORM(T, 1); break;    \
        case 2: LA_NORM(T, 2); break;    \
        case 4: LA_NORM(T, 4); break;    \
        case 8: LA_NORM(T, 8); break;    \
        default: LA_NORM(T, 0); break;   \
    }
    if (dtype == KA_F32) { LA_NORM_ALL(float) } else { LA_NORM_ALL(bf16_t) }
#undef LA_NORM_ALL
#undef LA_NORM
    KA_LAUNCH_CHECK();
    return 0;
}

// ----------------------------------------------------------------------------
// Every head of fp32 read-outs raw [n, H, dv] normalised by itself: out = o / sqrt(mean(o^2) + eps) * gain [dv] (shared by the
// heads) * silu(gate): a group of 16 lanes per (token, head).
// ----------------------------------------------------------------------------
template <typename T, bool VECTORS>
__global__ void __launch_bounds__(LA_THREADS)
heads_rmsnorm_kernel(const float* __restrict__ raw, const float* __restrict__ gain, const T* __restrict__ gate, long gate_stride,
                     T* __restrict__ out, long out_stride, long pairs, int H, int dv, float eps) {
    constexpr int LANES = 16;
    const long pair = (long)blockIdx.x * (LA_THREADS / LANES) + threadIdx.x / LANES;
    const int lane = threadIdx.x % LANES;
    const bool live = pair < pairs;
    const long t = live ? pair / H : 0;
    const int head = live ? (int)(pair % H) : 0;
    const float* o = raw + (t * H + head) * dv;
    const T* g = gate + t * gate_stride + (size_t)head * dv;
    T* dst = out + t * out_stride + (size_t)head * dv;
    float ss = 0.f;
    if constexpr (VECTORS) {
        for (int c = lane * 4; c < dv; c += LANES * 4) {
            const float4 v = *reinterpret_cast<const float4*>(o + c);
            ss += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
        }
    } else {
        for (int c = lane; c < dv; c += LANES) ss = fmaf(o[c], o[c], ss);
    }
    ss = ka_lanes_reduce<1, LANES>(ss, KaSum{});
    if (!live) return;
    const float r = 1.0f / sqrtf(ss / (float)dv + eps);
    if constexpr (VECTORS) {
        typedef __attribute__((ext_vector_type(4))) T vec;
        for (int c = lane * 4; c < dv; c += LANES * 4) {
            const float4 v = *reinterpret_cast<const float4*>(o + c), w = *reinterpret_cast<const float4*>(gain + c);
            const vec x = *reinterpret_cast<const vec*>(g + c);
            const float y[4] = {v.x * w.x, v.y * w.y, v.z * w.z, v.w * w.w};
            vec b;
#pragma unroll
            for (int e = 0; e < 4; ++e) b[e] = ka_from_float<T>(y[e] * r * la_act<T>(KA_ACT_SILU, ka_to_float(x[e])));
            *reinterpret_cast<vec*>(dst + c) = b;
        }
    } else {
        for (int c = lane; c < dv; c += LANES)
            dst[c] = ka_from_float<T>(o[c] * r * gain[c] * la_act<T>(KA_ACT_SILU, ka_to_float(g[c])));
    }
}

KA_API int ka_heads_rmsnorm(const float* raw, const float* gain, const void* gate, long gate_stride, void* out, long out_stride, int dtype,
                            int n, int H, int dv, float eps, hipStream_t stream) {
    const char* who = "ka_heads_rmsnorm";
    KA_CHECK(n >= 0 && H > 0 && dv > 0 && eps >= 0.f && gate_stride >= (long)H * dv && out_stride >= (long)H * dv, "%s: bad sizes", who);
    KA_CHECK(dtype == KA_F32 || dtype == KA_BF16, "%s: unsupported dtype %d", who, dtype);
    KA_CHECK(gain != nullptr && gate != nullptr, "%s: gains and gate missing", who);
    if (n == 0) return 0;
    const size_t align = dtype == KA_F32 ? 16 : 8;
    const bool vectors = dv % 4 == 0 && gate_stride % 4 == 0 && out_stride % 4 == 0 && (uintptr_t)raw % 16 == 0 && (uintptr_t)gain % 16 == 0 &&
                         (uintptr_t)gate % align == 0 && (uintptr_t)out % align == 0;
    const long pairs = (long)n * H;
    const dim3 grid(ka_cdiv(pairs, LA_THREADS / 16));
#define LA_HEADS(T, V) \
    hipLaunchKernelGGL((heads_rmsnorm_kernel<T, V>), grid, dim3(LA_THREADS), 0, stream, raw, gain, (const T*)gate, gate_stride, (T*)out, out_stride, pairs, H, dv, eps)
    if (dtype == KA_F32) { if (vectors) LA_HEADS(float, true); else LA_HEADS(float, false); }
    else { if (vectors) LA_HEADS(bf16_t, true); else LA_HEADS(bf16_t, false); }
#undef LA_HEADS
    KA_LAUNCH_CHECK();
    return 0;
}

// ----------------------------------------------------------------------------
// One token of a recurrence that forgets channel by channel, from the projected row to the input of the output projection in
// one launch: the decay's second linear z = W_a2 low + b and the decays, the head's state moved on by the token, the read-out, its
// norm, gain and gate. A workgroup takes a head of a row; a group of 16 lanes takes value channels, NV times four key channels
// a lane. The state is asked for before anything that it meets is computed. A row without a request gets zeros.
// ----------------------------------------------------------------------------
struct GatedStepArgs {
    const void* row;            // [n, stride]: the projected rows (row r: the token of row r)
    long stride;
    int at_q, at_k, at_v, at_gate, at_low, rank;
    const void* a2;             // [H d, rank]
    const float* a2_bias;       // [H d]
    const float* gain;          // [dv]
    float* state;               // [slots, state_stride]: S [H, dv, d]
    long state_stride;
    const int* row_slot;
    void* out;                  // [n, out_stride]
    long out_stride;
    int H, d, dv;
    float per_tau, q_scale, eps;
};

constexpr int LS_MAX_D = 256, LS_MAX_DV = 512, LS_MAX_RANK = 1024;

template <typename T, int NV>
__global__ void __launch_bounds__(LA_THREADS) gated_step_kernel(GatedStepArgs a) {
    constexpr int LANES = 16, GROUPS = LA_THREADS / LANES, AT_ONCE = 8 / NV;      // value channels of a group in flight
    __shared__ __attribute__((aligned(16))) float q_s[LS_MAX_D], k_s[LS_MAX_D], w_s[LS_MAX_D];
    __shared__ float low_s[LS_MAX_RANK], o_s[LS_MAX_DV], v_s[LS_MAX_DV], part[LA_THREADS / KA_WAVE];
    const int head = blockIdx.x, r = blockIdx.y, tid = threadIdx.x;
    const int d = a.d, dv = a.dv;
    const T* row = reinterpret_cast<const T*>(a.row) + (size_t)r * a.stride;
    T* out = reinterpret_cast<T*>(a.out) + (size_t)r * a.out_stride + (size_t)head * dv;
    const int slot = a.row_slot[r];
    if (slot < 0) {
        for (int j = tid; j < dv; j += LA_THREADS) out[j] = ka_from_float<T>(0.f);
        return;
    }
    const int group = tid / LANES, lane = tid % LANES;
    float* S = a.state + (size_t)slot * a.state_stride + (size_t)head * d * dv;
    float4 s[AT_ONCE][NV];
    auto fetch = [&](int j0) {
#pragma unroll
        for (int m = 0; m < AT_ONCE; ++m)
#pragma unroll
            for (int u = 0; u < NV; ++u) {
                const int j = j0 + m * GROUPS + group, i = (u * LANES + lane) * 4;
                s[m][u] = j < dv && i < d ? *reinterpret_cast<const float4*>(S + (size_t)j * d + i) : make_float4(0.f, 0.f, 0.f, 0.f);
            }
    };
    fetch(0);
    for (int c = tid; c < a.rank; c += LA_THREADS) low_s[c] = ka_to_float(row[a.at_low + c]);
    for (int i = tid; i < d; i += LA_THREADS) {
        q_s[i] = ka_to_float(row[a.at_q + head * d + i]) * a.q_scale;
        k_s[i] = ka_to_float(row[a.at_k + head * d + i]);
    }
    for (int j = tid; j < dv; j += LA_THREADS) v_s[j] = ka_to_float(row[a.at_v + head * dv + j]);
    __syncthreads();
    // (four lanes a key channel)
    for (int i0 = 0; i0 < d; i0 += LA_THREADS / 4) {
        const int i = min(i0 + tid / 4, d - 1);
        const T* w = reinterpret_cast<const T*>(a.a2) + ((size_t)head * d + i) * a.rank;
        float z = 0.f;
#pragma unroll 8
        for (int c = tid % 4; c < a.rank; c += 4) z = fmaf(ka_to_float(w[c]), low_s[c], z);
        z = ka_lanes_reduce<1, 4>(z, KaSum{}) + a.a2_bias[head * d + i];
        if (tid % 4 == 0) w_s[i] = ka_decay<sizeof(T) == 2>(z, a.per_tau);
    }
    __syncthreads();
    float4 q[NV], k[NV], w[NV];
#pragma unroll
    for (int u = 0; u < NV; ++u) {
        const int i = min((u * LANES + lane) * 4, d - 4);
        q[u] = *reinterpret_cast<const float4*>(q_s + i);
        k[u] = *reinterpret_cast<const float4*>(k_s + i);
        w[u] = *reinterpret_cast<const float4*>(w_s + i);
    }
    float ss = 0.f;
    for (int j0 = 0; j0 < dv; j0 += AT_ONCE * GROUPS) {
        if (j0 > 0) fetch(j0);
#pragma unroll
        for (int m = 0; m < AT_ONCE; ++m) {
            const int j = j0 + m * GROUPS + group;
            const float v = j < dv ? v_s[j] : 0.f;
            float acc = 0.f;
#pragma unroll
            for (int u = 0; u < NV; ++u) {
                const int i = (u * LANES + lane) * 4;
                if (i >= d) continue;
                float4& x = s[m][u];
                x.x = fmaf(w[u].x, x.x, k[u].x * v);
                x.y = fmaf(w[u].y, x.y, k[u].y * v);
                x.z = fmaf(w[u].z, x.z, k[u].z * v);
                x.w = fmaf(w[u].w, x.w, k[u].w * v);
                acc = fmaf(q[u].x, x.x, acc);
                acc = fmaf(q[u].y, x.y, acc);
                acc = fmaf(q[u].z, x.z, acc);
                acc = fmaf(q[u].w, x.w, acc);
                if (j < dv) *reinterpret_cast<float4*>(S + (size_t)j * d + i) = x;
            }
            acc = ka_lanes_reduce<1, LANES>(acc, KaSum{});
            if (lane == 0 && j < dv) {
                o_s[j] = acc;
                ss = fmaf(acc, acc, ss);
            }
        }
    }
    ss = ka_wave_sum(ss);
    if (tid % KA_WAVE == 0) part[tid / KA_WAVE] = ss;
    __syncthreads();
    float total = 0.f;
#pragma unroll
    for (int v = 0; v < LA_THREADS / KA_WAVE; ++v) total += part[v];
    const float scale = 1.0f / sqrtf(total / (float)dv + a.eps);
    for (int j = tid; j < dv; j += LA_THREADS)
        out[j] = ka_from_float<T>(o_s[j] * scale * a.gain[j] * la_act<T>(KA_ACT_SILU, ka_to_float(row[a.at_gate + head * dv + j])));
}

// Whether the kernel covers heads of these sizes: key channels in steps of four.
KA_API int ka_gated_step_supported(int d, int dv, int rank) {
    return d > 0 && d % 4 == 0 && d <= LS_MAX_D && dv > 0 && dv <= LS_MAX_DV && rank > 0 && rank <= LS_MAX_RANK ? 1 : 0;
}

KA_API int ka_gated_step(const void* row, long stride, int dtype, int at_q, int at_k, int at_v, int at_gate, int at_low, int rank, const void* a2,
                         const float* a2_bias, const float* gain, float tau, float q_scale, float eps, float* state, long state_stride,
                         const int* row_slot, void* out, long out_stride, int n, int H, int d, int dv, hipStream_t stream) {
    const char* who = "ka_gated_step";
    KA_CHECK(n >= 0 && n <= 65535 && H > 0 && ka_gated_step_supported(d, dv, rank), "%s: heads of %d x %d channels, a rank of %d are not covered", who, d, dv, rank);
    KA_CHECK(dtype == KA_F32 || dtype == KA_BF16, "%s: unsupported dtype %d", who, dtype);
    KA_CHECK(tau > 0.f && eps >= 0.f, "%s: a positive tau and an epsilon that is not negative", who);
    const long ends[5] = {at_q + (long)H * d, at_k + (long)H * d, at_v + (long)H * dv, at_gate + (long)H * dv, at_low + (long)rank};
    for (long end : ends) KA_CHECK(end <= stride, "%s: the projected rows are too short", who);
    KA_CHECK(at_q >= 0 && at_k >= 0 && at_v >= 0 && at_gate >= 0 && at_low >= 0 && out_stride >= (long)H * dv, "%s: bad columns", who);
    KA_CHECK(state_stride >= (long)H * d * dv && state_stride % 4 == 0 && (uintptr_t)state % 16 == 0, "%s: the state's rows must be 16-byte aligned", who);
    if (n == 0) return 0;
    const GatedStepArgs a{row, stride, at_q, at_k, at_v, at_gate, at_low, rank, a2, a2_bias, gain, state, state_stride, row_slot, out, out_stride,
                          H, d, dv, 1.f / tau, q_scale, eps};
#define LA_STEP(T)                                                                                                                            \
    if (d <= 64) hipLaunchKernelGGL((gated_step_kernel<T, 1>), dim3(H, n), dim3(LA_THREADS), 0, stream, a);       \
    else if (d <= 128) hipLaunchKernelGGL((gated_step_kernel<T, 2>), dim3(H, n), dim3(LA_THREADS), 0, stream, a); \
    else hipLaunchKernelGGL((gated_step_kernel<T, 4>), dim3(H, n), dim3(LA_THREADS), 0, stream, a)
    if (dtype == KA_F32) { LA_STEP(float); }
    else { LA_STEP(bf16_t); }
#undef LA_STEP
    KA_LAUNCH_CHECK();
    return 0;
}
