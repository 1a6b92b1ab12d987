// Kernels of a residual stream that is several copies (hyper-connections): x [n, S, dim] fp32. One launch stands between two
// sublayers: it writes the output y of the one before into the streams, all of them at once from the old ones,
//     x_t <- sum_s mix[s, t] x_s + out[t] y,
// reads what the next sublayer sees, u = sum_t into[t] x_t, and leaves that sublayer's norm of u in h. All arithmetic is fp32.
// What computes y is the caller's business: a load, or the weighted sum of a routed mixture's experts.
#include "ka_common.h"

constexpr int ST_THREADS = 256;
constexpr int ST_WAVES = ST_THREADS / KA_WAVE;
constexpr int ST_MAX_STREAMS = 16;

struct StreamArgs {
    float* x;                   // [rows of the stream, S, dim]
    const float* embedded;      // [n, dim]: every stream starts as this row (x is written only); null: x is read
    const float* mix;           // [S, S] from, to; null: nothing is written into the streams
    const float* out;           // [S]
    const float* into;          // [S]; null: the sum of the streams is read
    const int* rows;            // rows of x that are read (nothing is written then), all inside x; null: row i
    const float* gain;
    const float* bias;          // may be null
    float eps;
    int rms;                    // 0: layer norm, 1: root mean square alone
    void* h;                    // [n, dim]; null: nothing is read
    int h_bf16;
    int S, dim;
};

__device__ __forceinline__ float st_block_sum(float v, float* smem) {
    v = ka_wave_sum(v);
    __syncthreads();
    if (threadIdx.x % KA_WAVE == 0) smem[threadIdx.x / KA_WAVE] = v;
    __syncthreads();
    float total = 0.f;
#pragma unroll
    for (int w = 0; w < ST_WAVES; ++w) total += smem[w];
    return total;
}

__device__ __forceinline__ float4 st_fma4(float a, const float4& b, const float4& c) {
    return make_float4(fmaf(a, b.x, c.x), fmaf(a, b.y, c.y), fmaf(a, b.z, c.z), fmaf(a, b.w, c.w));
}

// S streams in registers, PIECES pieces of four channels a thread (dim a multiple of 4 and at most 4 PIECES ST_THREADS, rows
// 16-byte aligned). `piece(c)` gives y of the channels c .. c + 3.
template <int S, int PIECES, typename Piece>
__device__ __forceinline__ void st_step_regs(const StreamArgs& a, Piece piece, float* smem) {
    typedef __attribute__((ext_vector_type(4))) __bf16 st_bf16x4;
    const int i = blockIdx.x, tid = threadIdx.x, dim = a.dim;
    float* row = a.x + (size_t)(a.rows ? a.rows[i] : i) * S * dim;
    float m[S][S], o[S], in[S];
    const bool writes = a.mix != nullptr;
    if (writes) {
#pragma unroll
        for (int s = 0; s < S; ++s) {
#pragma unroll
            for (int t = 0; t < S; ++t) m[s][t] = a.mix[s * S + t];
            o[s] = a.out[s];
        }
    }
#pragma unroll
    for (int s = 0; s < S; ++s) in[s] = a.into ? a.into[s] : 1.f;
    float4 u[PIECES];
    float sum = 0.f;
    // (all that a few pieces need is asked for before anything is stored)
    constexpr int AT_ONCE = PIECES < 4 ? PIECES : 4;
#pragma unroll
    for (int p0 = 0; p0 < PIECES; p0 += AT_ONCE) {
        float4 v[AT_ONCE][S], y[AT_ONCE];
#pragma unroll
        for (int p = 0; p < AT_ONCE; ++p) {
            const int c = ((p0 + p) * ST_THREADS + tid) * 4;
            if (c >= dim) continue;
            if (a.embedded) {
                v[p][0] = *reinterpret_cast<const float4*>(a.embedded + (size_t)i * dim + c);
            } else {
#pragma unroll
                for (int s = 0; s < S; ++s) v[p][s] = *reinterpret_cast<const float4*>(row + (size_t)s * dim + c);
            }
            if (writes) y[p] = piece(c);
        }
#pragma unroll
        for (int p = 0; p < AT_ONCE; ++p) {
            const int c = ((p0 + p) * ST_THREADS + tid) * 4;
            float4& sums = u[p0 + p];
            sums = make_float4(0.f, 0.f, 0.f, 0.f);
            if (c >= dim) continue;
            if (a.embedded) {
#pragma unroll
                for (int s = 0; s < S; ++s) {
                    v[p][s] = v[p][0];
                    *reinterpret_cast<float4*>(row + (size_t)s * dim + c) = v[p][0];
                }
            }
            if (writes) {
#pragma unroll
                for (int t = 0; t < S; ++t) {
                    float4 w = make_float4(o[t] * y[p].x, o[t] * y[p].y, o[t] * y[p].z, o[t] * y[p].w);
#pragma unroll
                    for (int s = 0; s < S; ++s) w = st_fma4(m[s][t], v[p][s], w);
                    *reinterpret_cast<float4*>(row + (size_t)t * dim + c) = w;
                    sums = st_fma4(in[t], w, sums);
                }
            } else {
#pragma unroll
                for (int s = 0; s < S; ++s) sums = st_fma4(in[s], v[p][s], sums);
            }
            sum += (sums.x + sums.y) + (sums.z + sums.w);
        }
    }
    if (a.h == nullptr) return;
    const float mean = a.rms ? 0.f : st_block_sum(sum, smem) / (float)dim;
    float ss = 0.f;
#pragma unroll
    for (int p = 0; p < PIECES; ++p) {
        if ((p * ST_THREADS + tid) * 4 < dim) {
            u[p] = make_float4(u[p].x - mean, u[p].y - mean, u[p].z - mean, u[p].w - mean);
            ss += u[p].x * u[p].x + u[p].y * u[p].y + u[p].z * u[p].z + u[p].w * u[p].w;
        }
    }
    const float r = 1.0f / sqrtf(st_block_sum(ss, smem) / (float)dim + a.eps);
#pragma unroll
    for (int p = 0; p < PIECES; ++p) {
        const int c = (p * ST_THREADS + tid) * 4;
        if (c < dim) {
            const float4 g = *reinterpret_cast<const float4*>(a.gain + c);
            float4 v = make_float4(u[p].x * r * g.x, u[p].y * r * g.y, u[p].z * r * g.z, u[p].w * r * g.w);
            if (a.bias) {
                const float4 b = *reinterpret_cast<const float4*>(a.bias + c);
                v = make_float4(v.x + b.x, v.y + b.y, v.z + b.z, v.w + b.w);
            }
            if (a.h_bf16) {
                st_bf16x4 b;
                b[0] = (bf16_t)v.x;
                b[1] = (bf16_t)v.y;
                b[2] = (bf16_t)v.z;
                b[3] = (bf16_t)v.w;
                *reinterpret_cast<st_bf16x4*>(reinterpret_cast<bf16_t*>(a.h) + (size_t)i * dim + c) = b;
            } else {
                *reinterpret_cast<float4*>(reinterpret_cast<float*>(a.h) + (size_t)i * dim + c) = v;
            }
        }
    }
}

// Any number of streams up to ST_MAX_STREAMS, any dim. `one(c)` gives y of channel c.
template <typename One>
__device__ __forceinline__ void st_step_any(const StreamArgs& a, One one, float* smem) {
    const int i = blockIdx.x, tid = threadIdx.x, dim = a.dim, S = a.S;
    float* row = a.x + (size_t)(a.rows ? a.rows[i] : i) * S * dim;
    const bool writes = a.mix != nullptr;
    auto read = [&](int c) {
        float u = 0.f;
        for (int s = 0; s < S; ++s) u = fmaf(a.into ? a.into[s] : 1.f, row[(size_t)s * dim + c], u);
        return u;
    };
    float sum = 0.f;
    for (int c = tid; c < dim; c += ST_THREADS) {
        if (a.embedded) {
            const float e = a.embedded[(size_t)i * dim + c];
            for (int s = 0; s < S; ++s) row[(size_t)s * dim + c] = e;
        }
        if (writes) {
            float v[ST_MAX_STREAMS];
#pragma unroll
            for (int s = 0; s < ST_MAX_STREAMS; ++s) v[s] = s < S ? row[(size_t)s * dim + c] : 0.f;
            const float y = one(c);
            for (int t = 0; t < S; ++t) {
                float w = a.out[t] * y;
#pragma unroll
                for (int s = 0; s < ST_MAX_STREAMS; ++s)
                    if (s < S) w = fmaf(a.mix[s * S + t], v[s], w);
                row[(size_t)t * dim + c] = w;
            }
        }
        if (a.h) sum += read(c);              // (a thread reads its own writes)
    }
    if (a.h == nullptr) return;
    const float mean = a.rms ? 0.f : st_block_sum(sum, smem) / (float)dim;
    float ss = 0.f;
    for (int c = tid; c < dim; c += ST_THREADS) {
        const float u = read(c) - mean;
        ss += u * u;
    }
    const float r = 1.0f / sqrtf(st_block_sum(ss, smem) / (float)dim + a.eps);
    for (int c = tid; c < dim; c += ST_THREADS) {
        float v = (read(c) - mean) * r * a.gain[c];
        if (a.bias) v += a.bias[c];
        if (a.h_bf16) reinterpret_cast<bf16_t*>(a.h)[(size_t)i * dim + c] = (bf16_t)v;
        else reinterpret_cast<float*>(a.h)[(size_t)i * dim + c] = v;
    }
}

template <int S, int PIECES>
__global__ void __launch_bounds__(ST_THREADS) streams_step_kernel(StreamArgs a, const float* __restrict__ y) {
    __shared__ float smem[ST_WAVES];
    const float* yr = y ? y + (size_t)blockIdx.x * a.dim : nullptr;
    if constexpr (S > 0)
        st_step_regs<S, PIECES>(a, [&](int c) { return *reinterpret_cast<const float4*>(yr + c); }, smem);
    else
        st_step_any(a, [&](int c) { return yr[c]; }, smem);
}

// y = sum_k weights[t, k] * (chosen[t, k] < E ? pairs[t top + k] : h_in[t]) + sigmoid(shared_gate[t]) * shared[t], as
// ka_experts_combine makes it, in its order.
struct StreamExperts {
    const float* pairs;         // [n top, dim]
    const void* h_in;
    long h_stride;
    const int* chosen;
    const float* weights;
    int top, E;
    const float* shared;
    const float* shared_gate;
    long gate_stride;
};

template <typename T, int S, int PIECES>
__global__ void __launch_bounds__(ST_THREADS) streams_experts_kernel(StreamArgs a, StreamExperts e) {
    __shared__ float smem[ST_WAVES];
    const int t = blockIdx.x, dim = a.dim;
    const T* hp = reinterpret_cast<const T*>(e.h_in) + (size_t)t * e.h_stride;
    const float sg = e.shared ? (e.shared_gate ? 1.0f / (1.0f + expf(-e.shared_gate[(size_t)t * e.gate_stride])) : 1.f) : 0.f;
    if constexpr (S > 0) {
        st_step_regs<S, PIECES>(a, [&](int c) {
            float4 acc = make_float4(0.f, 0.f, 0.f, 0.f);
            // (four choices in flight; a choice without weights of its own has a row in `pairs` too, which is not used)
            for (int k0 = 0; k0 < e.top; k0 += 4) {
                float4 v[4];
                float w[4];
#pragma unroll
                for (int k = 0; k < 4; ++k) {
                    const size_t at = (size_t)t * e.top + min(k0 + k, e.top - 1);
                    w[k] = e.weights[at];
                    v[k] = *reinterpret_cast<const float4*>(e.pairs + at * dim + c);
                    if (e.chosen[at] >= e.E) v[k] = make_float4(ka_to_float(hp[c]), ka_to_float(hp[c + 1]), ka_to_float(hp[c + 2]), ka_to_float(hp[c + 3]));
                }
#pragma unroll
                for (int k = 0; k < 4; ++k)
                    if (k0 + k < e.top) acc = st_fma4(w[k], v[k], acc);
            }
            if (e.shared) acc = st_fma4(sg, *reinterpret_cast<const float4*>(e.shared + (size_t)t * dim + c), acc);
            return acc;
        }, smem);
    } else {
        st_step_any(a, [&](int c) {
            float acc = 0.f;
            for (int k = 0; k < e.top; ++k) {
                const float v = e.chosen[(size_t)t * e.top + k] < e.E ? e.pairs[((size_t)t * e.top + k) * dim + c] : ka_to_float(hp[c]);
                acc = fmaf(e.weights[(size_t)t * e.top + k], v, acc);
            }
            return e.shared ? fmaf(sg, e.shared[(size_t)t * dim + c], acc) : acc;
        }, smem);
    }
}

// Pieces of four channels a thread holds in the form with registers; 0: the general form.
static int st_pieces(const StreamArgs& a, const void* y, const void* shared) {
    const uintptr_t all = (uintptr_t)a.x | (uintptr_t)a.embedded | (uintptr_t)a.gain | (uintptr_t)a.bias | (uintptr_t)y | (uintptr_t)shared;
    if (a.S > 4 || a.dim % 4 != 0 || all % 16 != 0 || (uintptr_t)a.h % (a.h_bf16 ? 8 : 16) != 0) return 0;
    const int need = ka_cdiv(a.dim, 4 * ST_THREADS);
    for (int p : {1, 2, 4, 8})
        if (need <= p) return p;
    return 0;
}

#define ST_CASES(LAUNCH, S)          \
    switch (pieces) {                \
        case 1: LAUNCH(S, 1); break; \
        case 2: LAUNCH(S, 2); break; \
        case 4: LAUNCH(S, 4); break; \
        default: LAUNCH(S, 8); break;\
    }
#define ST_DISPATCH(LAUNCH)                       \
    if (pieces == 0) { LAUNCH(0, 0); }            \
    else if (a.S == 1) { ST_CASES(LAUNCH, 1) }    \
    else if (a.S == 2) { ST_CASES(LAUNCH, 2) }    \
    else if (a.S == 3) { ST_CASES(LAUNCH, 3) }    \
    else { ST_CASES(LAUNCH, 4) }

static int st_check(const char* who, const StreamArgs& a, int n, int h_dtype) {
    KA_CHECK(n >= 0 && a.S > 0 && a.S <= ST_MAX_STREAMS && a.dim > 0 && a.eps >= 0.f, "%s: bad sizes (%d streams of %d)", who, a.S, a.dim);
    KA_CHECK(h_dtype == KA_F32 || h_dtype == KA_BF16, "%s: unsupported dtype %d", who, h_dtype);
    KA_CHECK((a.mix == nullptr) == (a.out == nullptr), "%s: writing needs both mix and out", who);
    KA_CHECK(a.h == nullptr || a.gain != nullptr, "%s: the norm needs its gains", who);
    KA_CHECK(a.rows == nullptr || (a.mix == nullptr && a.embedded == nullptr), "%s: chosen rows are only read", who);
    return 0;
}

KA_API int ka_streams_step(float* x, const float* embedded, const float* y, const float* mix, const float* out, const float* into,
                           const int* rows, const float* gain, const float* bias, float eps, int rms, void* h, int h_dtype, int n, int S,
                           int dim, hipStream_t stream) {
    const char* who = "ka_streams_step";
    const StreamArgs a{x, embedded, mix, out, into, rows, gain, bias, eps, rms, h, h_dtype == KA_BF16, S, dim};
    if (const int status = st_check(who, a, n, h_dtype)) return status;
    KA_CHECK((mix == nullptr) == (y == nullptr), "%s: writing needs a sublayer's output", who);
    if (n == 0) return 0;
    const int pieces = st_pieces(a, y, nullptr);
#define ST_LAUNCH(S_, P_) hipLaunchKernelGGL((streams_step_kernel<S_, P_>), dim3(n), dim3(ST_THREADS), 0, stream, a, y)
    ST_DISPATCH(ST_LAUNCH)
#undef ST_LAUNCH
    KA_LAUNCH_CHECK();
    return 0;
}

KA_API int ka_streams_experts(float* x, const float* pairs, const void* h_in, long h_stride, int dtype, const int* chosen,
                              const float* weights, int top, int E, const float* shared, const float* shared_gate, long gate_stride,
                              const float* mix, const float* out, const float* into, const float* gain, const float* bias, float eps,
                              int rms, void* h, int h_dtype, int n, int S, int dim, hipStream_t stream) {
    const char* who = "ka_streams_experts";
    const StreamArgs a{x, nullptr, mix, out, into, nullptr, gain, bias, eps, rms, h, h_dtype == KA_BF16, S, dim};
    if (const int status = st_check(who, a, n, h_dtype)) return status;
    KA_CHECK(mix != nullptr && top > 0 && h_stride >= dim, "%s: bad sizes", who);
    KA_CHECK(dtype == KA_F32 || dtype == KA_BF16, "%s: unsupported dtype %d", who, dtype);
    if (n == 0) return 0;
    const StreamExperts e{pairs, h_in, h_stride, chosen, weights, top, E, shared, shared_gate, gate_stride};
    const int pieces = st_pieces(a, pairs, shared);
#define ST_LAUNCH_F32(S_, P_) hipLaunchKernelGGL((streams_experts_kernel<float, S_, P_>), dim3(n), dim3(ST_THREADS), 0, stream, a, e)
#define ST_LAUNCH_BF16(S_, P_) hipLaunchKernelGGL((streams_experts_kernel<bf16_t, S_, P_>), dim3(n), dim3(ST_THREADS), 0, stream, a, e)
    if (dtype == KA_F32) { ST_DISPATCH(ST_LAUNCH_F32) } else { ST_DISPATCH(ST_LAUNCH_BF16) }
#undef ST_LAUNCH_F32
#undef ST_LAUNCH_BF16
    KA_LAUNCH_CHECK();
    return 0;
}
