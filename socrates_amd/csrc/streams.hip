// Kernels of decoders that keep several copies of the residual stream: the embedding with learned positions spread
// over the copies, and what stands between two branches: the branches' results added up, the new copies from the old
// ones, and the combination of the copies that the next branch reads, normed.
//
// The copies, the sums and the norm's statistics are float32 whatever the compute dtype; a value is rounded once,
// where it is stored in the compute dtype.
#include "common.h"

__device__ __forceinline__ void put4(float* p, const float (&x)[4]) { *reinterpret_cast<float4*>(p) = make_float4(x[0], x[1], x[2], x[3]); }
__device__ __forceinline__ void put4(bf16* p, const float (&x)[4]) {
    *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(x[0], x[1]), pack_bf16x2(x[2], x[3]));
}
template <typename T, int V> __device__ __forceinline__ void put(T* p, const float (&x)[V]) {
    if constexpr (V == 4) put4(p, x);
    else {
#pragma unroll
        for (int e = 0; e < V; ++e) p[e] = from_float<T>(x[e]);
    }
}

// ---- scale * table[id] + position_table[position], into every copy -------------------------------------------
// out float32 [N, S, d]; position_table [rows, d] or null. Ids and positions are clamped to their tables.
template <typename W>
__global__ void embedding_streams_kernel(const int* __restrict__ ids, const W* __restrict__ table, float scale,
                                         const int* __restrict__ positions, const W* __restrict__ position_table, int rows,
                                         float* __restrict__ out, int S, int d, int vocab) {
    const int n = blockIdx.y;
    const size_t src = (size_t)min(max(ids[n], 0), vocab - 1) * d;
    const size_t pos = position_table ? (size_t)min(max(positions[n], 0), rows - 1) * d : 0;
    for (int c = blockIdx.x * blockDim.x + threadIdx.x; c < d; c += gridDim.x * blockDim.x) {
        float v = to_float(table[src + c]) * scale;
        if (position_table) v += to_float(position_table[pos + c]);
        for (int s = 0; s < S; ++s) out[((size_t)n * S + s) * d + c] = v;
    }
}

SOC_EXPORT int soc_embedding_streams(const int* ids, const void* table, float scale, const int* positions,
                                     const void* position_table, int rows, float* out, int N, int S, int d, int vocab, int dtype,
                                     hipStream_t stream) {
    if (N <= 0) return 0;
    if (N > 65535 || S < 1 || d < 1 || vocab < 1 || (position_table && (rows < 1 || !positions))) return (int)hipErrorInvalidValue;
    const dim3 grid((d + 255) / 256 < 16 ? (d + 255) / 256 : 16, N);
    if (dtype == 0)
        hipLaunchKernelGGL(embedding_streams_kernel<float>, grid, dim3(256), 0, stream, ids, (const float*)table, scale, positions,
                           (const float*)position_table, rows, out, S, d, vocab);
    else
        hipLaunchKernelGGL(embedding_streams_kernel<bf16>, grid, dim3(256), 0, stream, ids, (const bf16*)table, scale, positions,
                           (const bf16*)position_table, rows, out, S, d, vocab);
    return soc_last_error();
}

// ---- close a branch, open the next ---------------------------------------------------------------------------
// One result that enters a branch's sum, times ``scale``: [N, d] in the compute dtype (parts 0, or float32 with parts
// 1), float32 partial sums [parts, N, d], or (top > 0) the experts' results float32 by place: the sum over r of
// weight[n, r] * y[place[n, r]], a place below 0 standing for row n of ``through`` (compute dtype, [N, d]).
struct StreamIn {
    const void* y;
    int parts;
    const int* place;
    const float* weight;
    int top;
    const void* through;
    float scale;
};

template <typename T, int V>
__device__ __forceinline__ void stream_in(const StreamIn& b, int n, size_t total, int d, int c, float (&acc)[V], bool first) {
    float x[V];
    if (b.top > 0) {
#pragma unroll
        for (int e = 0; e < V; ++e) x[e] = 0.f;
        float same[V];                                          // (read once, so that the loads below need no branch)
#pragma unroll
        for (int e = 0; e < V; ++e) same[e] = 0.f;
        if (b.through) VecLoad<T, V>::load((const T*)b.through + (size_t)n * d + c, same);
        for (int r0 = 0; r0 < b.top; r0 += 4) {                 // four at a time: their loads are on the way together
            float t[4][V], w[4];
            int at[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const size_t i = (size_t)n * b.top + min(r0 + r, b.top - 1);
                at[r] = b.place[i];
                w[r] = b.weight[i];
            }
#pragma unroll
            for (int r = 0; r < 4; ++r) VecLoad<float, V>::load((const float*)b.y + (size_t)max(at[r], 0) * d + c, t[r]);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                if (r0 + r < b.top) {
#pragma unroll
                    for (int e = 0; e < V; ++e) x[e] = fmaf(w[r], at[r] >= 0 ? t[r][e] : same[e], x[e]);
                }
            }
        }
    } else if (b.parts > 0) {
        VecLoad<float, V>::load((const float*)b.y + (size_t)n * d + c, x);
        for (int s = 1; s < b.parts; ++s) {
            float t[V];
            VecLoad<float, V>::load((const float*)b.y + (size_t)s * total + (size_t)n * d + c, t);
#pragma unroll
            for (int e = 0; e < V; ++e) x[e] += t[e];
        }
    } else {
        VecLoad<T, V>::load((const T*)b.y + (size_t)n * d + c, x);
    }
#pragma unroll
    for (int e = 0; e < V; ++e) acc[e] = first ? b.scale * x[e] : fmaf(b.scale, x[e], acc[e]);
}

// The norm behind the combination (gain null: none): over the root mean square, or with ``centred`` the mean off first
// and the bias (null: none) added.
struct StreamNorm {
    const float* gain;
    const float* bias;
    float eps;
    int centred;
};

// One workgroup per row of out. x float32 [N, S, d]. With a.y: the old copies x_s and y = a (+ b) give
// x_t <- sum_s mix[s, t] x_s + out_w[t] y (mix null: x_t <- x_t + y). Then u = sum_t read[t] x_t (read null: plain
// sum), normed into out (no gain: nothing more). Without a.y nothing is written to x, and rows (null: all) selects the
// rows of x that are read. NT threads, PER pieces of V elements per thread, the combination staying in registers; PER 0: any number of
// pieces, the combination in LDS (d floats, every thread its own).
template <typename T, int SP, int V, int PER, int NT>
__global__ void __launch_bounds__(NT)
streams_kernel(float* __restrict__ x, int S, StreamIn a, StreamIn b, const float* __restrict__ mix, const float* __restrict__ out_w,
               const float* __restrict__ read, StreamNorm norm, const int* __restrict__ rows, T* __restrict__ out, int N, int d) {
    __shared__ float scratch[16];
    extern __shared__ float held[];
    const int n = rows ? rows[blockIdx.x] : (int)blockIdx.x;
    const size_t total = (size_t)N * d;
    float* row = x + (size_t)n * S * d;
    float kept[PER > 0 ? PER : 1][V], sum = 0.f;
    auto combine = [&](int c, float (&u)[V]) {
#pragma unroll
        for (int e = 0; e < V; ++e) u[e] = 0.f;
        float old[SP][V];
#pragma unroll
        for (int s = 0; s < SP; ++s)
            if (s < S) VecLoad<float, V>::load(row + (size_t)s * d + c, old[s]);
        if (a.y) {
            float y[V];
            stream_in<T, V>(a, n, total, d, c, y, true);
            if (b.y) stream_in<T, V>(b, n, total, d, c, y, false);
#pragma unroll
            for (int t = 0; t < SP; ++t) {
                if (t < S) {
                    float v[V];
                    const float w = mix ? out_w[t] : 1.f;
#pragma unroll
                    for (int e = 0; e < V; ++e) v[e] = w * y[e];
#pragma unroll
                    for (int s = 0; s < SP; ++s) {
                        if (s < S) {
                            const float m = mix ? mix[s * S + t] : (s == t ? 1.f : 0.f);
#pragma unroll
                            for (int e = 0; e < V; ++e) v[e] = fmaf(m, old[s][e], v[e]);
                        }
                    }
                    put<float, V>(row + (size_t)t * d + c, v);
                    const float r = read ? read[t] : 1.f;
#pragma unroll
                    for (int e = 0; e < V; ++e) u[e] = fmaf(r, v[e], u[e]);
                }
            }
        } else {
#pragma unroll
            for (int t = 0; t < SP; ++t) {
                if (t < S) {
                    const float r = read ? read[t] : 1.f;
#pragma unroll
                    for (int e = 0; e < V; ++e) u[e] = fmaf(r, old[t][e], u[e]);
                }
            }
        }
#pragma unroll
        for (int e = 0; e < V; ++e) sum += u[e];
    };
    // every piece of the combination, wherever it is kept
    auto pieces = [&](auto&& f) {
        if constexpr (PER > 0) {
#pragma unroll
            for (int i = 0; i < PER; ++i) {
                const int c = (threadIdx.x + i * NT) * V;
                if (c < d) f(c, kept[i]);
            }
        } else {
            for (int c = threadIdx.x * V; c < d; c += NT * V) {
                float u[V];
#pragma unroll
                for (int e = 0; e < V; ++e) u[e] = held[c + e];
                f(c, u);
#pragma unroll
                for (int e = 0; e < V; ++e) held[c + e] = u[e];
            }
        }
    };
    pieces([&](int c, float (&u)[V]) { combine(c, u); });
    if (!norm.gain) return;
    const float mean = norm.centred ? block_sum(sum, scratch) / (float)d : 0.f;
    float ss = 0.f;
    pieces([&](int, float (&u)[V]) {
#pragma unroll
        for (int e = 0; e < V; ++e) {
            u[e] -= mean;
            ss = fmaf(u[e], u[e], ss);
        }
    });
    const float inv = 1.f / sqrtf(block_sum(ss, scratch) / (float)d + norm.eps);
    T* dst = out + (size_t)blockIdx.x * d;
    pieces([&](int c, float (&u)[V]) {
        float g[V], h[V];
        VecLoad<float, V>::load(norm.gain + c, g);
        if (norm.bias) VecLoad<float, V>::load(norm.bias + c, h);
#pragma unroll
        for (int e = 0; e < V; ++e) g[e] = norm.bias ? fmaf(u[e] * inv, g[e], h[e]) : u[e] * inv * g[e];
        put<T, V>(dst + c, g);
    });
}

template <typename T, int SP>
static int launch_streams(float* x, int S, const StreamIn& a, const StreamIn& b, const float* mix, const float* out_w, const float* read,
                          const StreamNorm& norm, const int* rows, void* out, int N, int n_out, int d, hipStream_t stream) {
#define SOC_ST(SPV, V, PER, NT)                                                                                                      \
    hipLaunchKernelGGL((streams_kernel<T, SPV, V, PER, NT>), dim3(n_out), dim3(NT), (PER) ? 0 : d * sizeof(float), stream, x, S, a, b, mix, \
                       out_w, read, norm, rows, (T*)out, N, d)
    if (d > 16000) return (int)hipErrorInvalidValue;            // (what LDS holds)
    if constexpr (SP <= 4) {
        if (d % 4 == 0 && d <= 1024) { SOC_ST(SP, 4, 1, 256); return soc_last_error(); }
        // (few rows: a row's pieces side by side, not one behind the other)
        if (d % 4 == 0 && d <= 2048 && n_out <= 512) { SOC_ST(SP, 4, 1, 512); return soc_last_error(); }
        if (d % 4 == 0 && d <= 4096 && n_out <= 512) { SOC_ST(SP, 4, 1, 1024); return soc_last_error(); }
        if (d % 4 == 0 && d <= 2048) { SOC_ST(SP, 4, 2, 256); return soc_last_error(); }
        if (d % 4 == 0 && d <= 3072) { SOC_ST(SP, 4, 3, 256); return soc_last_error(); }
        if (d % 4 == 0 && d <= 4096) { SOC_ST(SP, 4, 4, 256); return soc_last_error(); }
    }
    constexpr int SPG = SP <= 4 ? 4 : 16;
    if (d % 4 == 0) SOC_ST(SPG, 4, 0, 256);
    else SOC_ST(SPG, 1, 0, 256);
#undef SOC_ST
    return soc_last_error();
}

SOC_EXPORT int soc_streams(float* x, int S, const void* y1, int parts1, const int* place1, const float* weight1, int top1,
                           const void* through1, float scale1, const void* y2, int parts2, const int* place2, const float* weight2,
                           int top2, const void* through2, float scale2, const float* mix, const float* out_w, const float* read,
                           const float* gain, const float* bias, float eps, int centred, const int* rows, void* out, int N, int n_out,
                           int d, int dtype, hipStream_t stream) {
    if (n_out <= 0) return 0;
    if (S < 1 || S > 16 || d < 1 || parts1 < 0 || parts2 < 0 || (top1 > 0 && (!place1 || !weight1)) || (top2 > 0 && (!place2 || !weight2)) ||
        (mix && !out_w) || (gain && !out) || (!gain && !y1) || (y2 && !y1) || (y1 && (rows || n_out != N)))
        return (int)hipErrorInvalidValue;
    const StreamIn a{y1, parts1, place1, weight1, top1, through1, scale1}, b{y2, parts2, place2, weight2, top2, through2, scale2};
    const StreamNorm norm{gain, bias, eps, centred};
#define SOC_STREAMS(SP) return dtype == 0 ? launch_streams<float, SP>(x, S, a, b, mix, out_w, read, norm, rows, out, N, n_out, d, stream) \
                                          : launch_streams<bf16, SP>(x, S, a, b, mix, out_w, read, norm, rows, out, N, n_out, d, stream)
    if (S == 1) SOC_STREAMS(1);
    if (S == 2) SOC_STREAMS(2);
    if (S <= 4) SOC_STREAMS(4);
    SOC_STREAMS(16);
#undef SOC_STREAMS
}
