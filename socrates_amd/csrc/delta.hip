// The gated delta rule: what prepares it (short causal convolutions with silu, unit vectors, decays and step sizes)
// and the recurrence itself, S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q per head.
//
// Everything behind the projections is float32; values alone are rounded to the compute dtype between the two kernels.
#include "common.h"
#include "recurrent.h"

__device__ __forceinline__ float dl_sigmoid(float x) { return 1.f / (1.f + expf(-x)); }

// ---- convolutions, activations, unit vectors, gates --------------------------------------------------------------
// x: rows of ldx elements that hold, from column col on, C = 2 G D + H Dv channels: q (G heads of D), k (G of D), v
// (H of Dv). Each channel passes a causal convolution of ``taps`` taps (taps_w [C, taps], the last one the current
// token's; inputs before the step's first token from the row's state [taps - 1, C] at ``offset``, which then becomes
// the step's last taps - 1 inputs) and silu. q and k become unit vectors per head, q also times q_scale: qk float32
// [N, 2, G, Dp], zeros behind D. v in the compute dtype [N, H Dv]. z float32 [N, 2 H] holds the logits of beta and,
// behind them, of the decay: gates float32 [N, H, 2] = (g, beta), g = exp(-exp(a_log) softplus(z + dt_bias)).
// Grid (2 G + H + 1 roles, chunks of DL_CHUNK tokens, sequences). A wave takes DL_RUN tokens in a row of its role's vector:
// with TAPS > 0 (the number of taps, up to 4) it loads all their inputs at once, each once; TAPS 0: any number of taps,
// token by token. Only a sequence's first chunk reads and writes the state (taps - 1 <= DL_CHUNK).
constexpr int DL_CHUNK = 32, DL_RUN = 8;

template <typename T, int TAPS, int NJ>
__global__ void __launch_bounds__(256)
delta_prepare_kernel(const T* __restrict__ x, int ldx, int col, int G, int H, int D, int Dv, int Dp, const float* __restrict__ taps_w,
                     int taps, float q_scale, float unit_eps, const float* __restrict__ z, const float* __restrict__ a_log,
                     const float* __restrict__ dt_bias, float* __restrict__ state, size_t stride, int offset,
                     const int* __restrict__ seq_qstart, const int* __restrict__ seq_rows, float* __restrict__ qk, T* __restrict__ v_out,
                     float* __restrict__ gates) {
    const int role = blockIdx.x, seq = blockIdx.z;
    const int lo = seq_qstart[seq], hi = seq_qstart[seq + 1];
    const int first = lo + blockIdx.y * DL_CHUNK;
    if (first >= hi) return;
    const int last = min(first + DL_CHUNK, hi);
    if (role == 2 * G + H) {                                    // the gates
        for (int e = threadIdx.x; e < (last - first) * H; e += blockDim.x) {
            const int n = first + e / H, h = e % H;
            const float u = z[(size_t)n * 2 * H + H + h] + dt_bias[h];
            const float step = fmaxf(u, 0.f) + log1pf(expf(-fabsf(u)));
            *reinterpret_cast<float2*>(gates + ((size_t)n * H + h) * 2) =
                make_float2(expf(-expf(a_log[h]) * step), dl_sigmoid(z[(size_t)n * 2 * H + h]));
        }
        return;
    }
    const bool is_v = role >= 2 * G;
    const int dim = is_v ? Dv : D, C = 2 * G * D + H * Dv;
    const int c0 = is_v ? 2 * G * D + (role - 2 * G) * Dv : role * D;      // first channel of the role's vector
    const int lane = threadIdx.x % SOC_WAVE, waves = blockDim.x / SOC_WAVE, back = taps - 1;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / SOC_WAVE);
    float* kept = state + (size_t)seq_rows[seq] * stride + offset;
    auto channel = [&](int n, int c) {
        float y = 0.f;
        for (int j = 0; j < taps; ++j) {
            const int idx = n - lo - back + j;                  // among the step's tokens of this sequence
            const float in = idx >= 0 ? to_float(x[(size_t)(lo + idx) * ldx + col + c]) : kept[(size_t)(back + idx) * C + c];
            y = fmaf(taps_w[(size_t)c * taps + j], in, y);
        }
        return y * dl_sigmoid(y);
    };
    if constexpr (TAPS > 0) {
        // pieces of 64 NJ channels (a q or k vector is one piece: its norm is taken of the wave's registers)
        const int n0 = first + wave * DL_RUN, n1 = min(n0 + DL_RUN, last);
        for (int i0 = 0; n0 < n1 && i0 < dim; i0 += 64 * NJ) {
            float in[DL_RUN + TAPS - 1][NJ], w[NJ][TAPS];
            // (every load stands on its own, with what lies outside the step redirected to a row of it: no branches)
#pragma unroll
            for (int r = 0; r < DL_RUN + TAPS - 1; ++r) {
                const T* row = x + (size_t)min(max(n0 - back + r, lo), n1 - 1) * ldx + col + c0;
#pragma unroll
                for (int j = 0; j < NJ; ++j) in[r][j] = to_float(row[min(i0 + lane + 64 * j, dim - 1)]);
            }
            if (n0 - lo < back) {                               // the sequence's first tokens: inputs of earlier steps
#pragma unroll
                for (int r = 0; r < TAPS - 1; ++r) {
                    const int idx = n0 - lo - back + r;
                    if (idx < 0) {
#pragma unroll
                        for (int j = 0; j < NJ; ++j) in[r][j] = kept[(size_t)(back + idx) * C + c0 + min(i0 + lane + 64 * j, dim - 1)];
                    }
                }
            }
#pragma unroll
            for (int j = 0; j < NJ; ++j) {
#pragma unroll
                for (int k = 0; k < TAPS; ++k) {
                    const int i = i0 + lane + 64 * j;
                    const float t = taps_w[(size_t)(c0 + min(i, dim - 1)) * TAPS + k];
                    w[j][k] = i < dim ? t : 0.f;                // (channels beyond the vector come out as zeros)
                }
            }
#pragma unroll
            for (int r = 0; r < DL_RUN; ++r) {
                if (n0 + r < n1) {
                    float y[NJ], ss = 0.f;
#pragma unroll
                    for (int j = 0; j < NJ; ++j) {
                        float a = 0.f;
#pragma unroll
                        for (int k = 0; k < TAPS; ++k) a = fmaf(w[j][k], in[r + k][j], a);
                        y[j] = a * dl_sigmoid(a);
                        ss = fmaf(y[j], y[j], ss);
                    }
                    const size_t n = n0 + r;
                    if (is_v) {
#pragma unroll
                        for (int j = 0; j < NJ; ++j) {
                            const int i = i0 + lane + 64 * j;
                            if (i < dim) v_out[n * H * Dv + (size_t)(role - 2 * G) * Dv + i] = from_float<T>(y[j]);
                        }
                    } else {
                        const float inv = 1.f / sqrtf(wave_sum(ss) + unit_eps) * (role < G ? q_scale : 1.f);
                        float* dst = qk + (n * 2 * G + role) * Dp;
#pragma unroll
                        for (int j = 0; j < NJ; ++j)
                            if (lane + 64 * j < Dp) dst[lane + 64 * j] = y[j] * inv;
                    }
                }
            }
        }
    } else
    for (int n = first + wave; n < last; n += waves) {
        if (is_v) {
            for (int i = lane; i < dim; i += SOC_WAVE) v_out[(size_t)n * H * Dv + (role - 2 * G) * Dv + i] = from_float<T>(channel(n, c0 + i));
        } else {
            float y[4], ss = 0.f;                               // D <= 256
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int i = lane + j * SOC_WAVE;
                y[j] = i < dim ? channel(n, c0 + i) : 0.f;
                ss = fmaf(y[j], y[j], ss);
            }
            const float inv = 1.f / sqrtf(wave_sum(ss) + unit_eps) * (role < G ? q_scale : 1.f);
            float* dst = qk + ((size_t)n * 2 * G + role) * Dp;
#pragma unroll
            for (int j = 0; j < 4; ++j)
                if (lane + j * SOC_WAVE < Dp) dst[lane + j * SOC_WAVE] = y[j] * inv;
        }
    }
    if (first == lo && back > 0) {
        __syncthreads();                                        // every wave has read what it needs of the state
        const int len = hi - lo;
        for (int i = threadIdx.x; i < dim; i += blockDim.x) {
            const int c = c0 + i;
            for (int j = 0; j < back; ++j) {                    // ascending: entry j + len is read before it is written
                const int idx = len - back + j;
                kept[(size_t)j * C + c] = idx >= 0 ? to_float(x[(size_t)(lo + idx) * ldx + col + c]) : kept[(size_t)(j + len) * C + c];
            }
        }
    }
}

SOC_EXPORT int soc_delta_prepare(const void* x, int ldx, int col, int G, int H, int D, int Dv, int Dp, const float* taps_w, int taps,
                                 float q_scale, float unit_eps, const float* z, const float* a_log, const float* dt_bias, float* state,
                                 long long stride, int offset, const int* seq_qstart, const int* seq_rows, float* qk, void* v_out,
                                 float* gates, int n_seqs, int max_q_len, int dtype, hipStream_t stream) {
    if (n_seqs <= 0) return 0;
    if (G < 1 || H < 1 || H % G || D < 1 || D > 256 || Dv < 1 || Dp < D || Dp > 256 || taps < 1 || taps - 1 > DL_CHUNK || n_seqs > 65535 ||
        max_q_len < 1)
        return (int)hipErrorInvalidValue;
    const dim3 grid(2 * G + H + 1, (max_q_len + DL_CHUNK - 1) / DL_CHUNK, n_seqs), block(max_q_len == 1 ? 64 : 256);
#define SOC_DP(T, TAPS, NJ)                                                                                                      \
    hipLaunchKernelGGL((delta_prepare_kernel<T, TAPS, NJ>), grid, block, 0, stream, (const T*)x, ldx, col, G, H, D, Dv, Dp, taps_w, taps, \
                       q_scale, unit_eps, z, a_log, dt_bias, state, (size_t)stride, offset, seq_qstart, seq_rows, qk, (T*)v_out, gates)
#define SOC_DP_T(T)                                                                                                     \
    if (taps == 4) { if (D <= 64) SOC_DP(T, 4, 1); else if (D <= 128) SOC_DP(T, 4, 2); else SOC_DP(T, 4, 4); }          \
    else if (taps == 3) { if (D <= 128) SOC_DP(T, 3, 2); else SOC_DP(T, 3, 4); }                                        \
    else if (taps == 2) { if (D <= 128) SOC_DP(T, 2, 2); else SOC_DP(T, 2, 4); }                                        \
    else SOC_DP(T, 0, 4);
    if (dtype == 0) { SOC_DP_T(float) } else { SOC_DP_T(bf16) }
#undef SOC_DP_T
#undef SOC_DP
    return soc_last_error();
}

// ---- the walk ------------------------------------------------------------------------------------------------------
// A workgroup owns 16 columns of one head's state, a wave four of them, and the 16 lanes of a row share a column: lane
// p holds the keys 64 j + 4 p .. + 3 in registers, so S^T k and S^T q are sums over a row of lanes (DPP, no LDS) and a
// column's part of the state [H, Dv, D] is contiguous in memory. Tokens go in batches staged through LDS with the
// next batch's loads in flight. out float32 [N, H Dv].
__device__ __forceinline__ float row16_sum(float v) {
    v += soc_dpp<SOC_DPP_XOR1>(v);
    v += soc_dpp<SOC_DPP_XOR2>(v);
    v += soc_dpp<SOC_DPP_HALF_MIRROR>(v);
    v += soc_dpp<SOC_DPP_ROW_MIRROR>(v);
    return v;
}

template <typename T, int NJ>
__global__ void __launch_bounds__(256)
delta_walk_kernel(const float* __restrict__ qk, const T* __restrict__ v, const float* __restrict__ gates, int G, int H, int D, int Dv,
                  float* __restrict__ state, size_t stride, int offset, const int* __restrict__ seq_qstart,
                  const int* __restrict__ seq_rows, float* __restrict__ out) {
    constexpr int DK = 64 * NJ, TB = NJ <= 2 ? 16 : 8, CW = 16, PIECES = TB * 2 * DK / 4, STAGE = PIECES / 256;
    static_assert(PIECES % 256 == 0, "whole rounds of 16-byte pieces");
    __shared__ __attribute__((aligned(16))) float sqk[2][TB][2][DK];
    __shared__ float sv[2][TB][CW], so[TB][CW];
    __shared__ float2 sg[2][TB];
    const int blocks = (Dv + CW - 1) / CW;
    const int head = blockIdx.x / blocks, seq = blockIdx.y, tid = threadIdx.x, kv = head / (H / G);
    const int lo = seq_qstart[seq], hi = seq_qstart[seq + 1];
    if (lo >= hi) return;
    const int col0 = (blockIdx.x % blocks) * CW, cl = tid / 16, p = tid % 16, col = col0 + cl;
    const bool live = col < Dv, vec = D % 4 == 0;
    float* S = state + (size_t)seq_rows[seq] * stride + offset + ((size_t)head * Dv + (live ? col : 0)) * D;
    float s[NJ][4];
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
        const int i = 64 * j + 4 * p;
        if (live && vec && i < D) {
            const float4 t = *reinterpret_cast<const float4*>(S + i);
            s[j][0] = t.x; s[j][1] = t.y; s[j][2] = t.z; s[j][3] = t.w;
        } else {
#pragma unroll
            for (int e = 0; e < 4; ++e) s[j][e] = live && i + e < D ? S[i + e] : 0.f;
        }
    }
    float4 fqk[STAGE];
    float fv = 0.f;
    float2 fg = make_float2(1.f, 0.f);
    auto fetch = [&](int n0) {
#pragma unroll
        for (int r = 0; r < STAGE; ++r) {
            const int e = tid + r * 256, t = e / (2 * DK / 4), which = e / (DK / 4) % 2, i = e % (DK / 4);
            fqk[r] = n0 + t < hi ? reinterpret_cast<const float4*>(qk + (((size_t)(n0 + t) * 2 + which) * G + kv) * DK)[i]
                                 : make_float4(0.f, 0.f, 0.f, 0.f);
        }
        const int t = tid / CW, c = col0 + tid % CW;
        if (t < TB) fv = n0 + t < hi && c < Dv ? to_float(v[(size_t)(n0 + t) * H * Dv + (size_t)head * Dv + c]) : 0.f;
        if (tid < TB) fg = n0 + tid < hi ? reinterpret_cast<const float2*>(gates)[(size_t)(n0 + tid) * H + head] : make_float2(1.f, 0.f);
    };
    auto land = [&](int buf) {
#pragma unroll
        for (int r = 0; r < STAGE; ++r) reinterpret_cast<float4*>(&sqk[buf][0][0][0])[tid + r * 256] = fqk[r];
        if (tid / CW < TB) sv[buf][tid / CW][tid % CW] = fv;
        if (tid < TB) sg[buf][tid] = fg;
    };
    fetch(lo);
    land(0);
    lds_barrier();
    int buf = 0;
    for (int n0 = lo; n0 < hi; n0 += TB, buf ^= 1) {
        const int nb = min(TB, hi - n0);
        const bool more = n0 + TB < hi;
        if (more) fetch(n0 + TB);
        auto token = [&](int t) {
            const float2 gb = sg[buf][t];
            float kk[NJ][4], qq[NJ][4], d0 = 0.f, d1 = 0.f;
#pragma unroll
            for (int j = 0; j < NJ; ++j) {
                VecLoad<float, 4>::load(&sqk[buf][t][1][64 * j + 4 * p], kk[j]);
                VecLoad<float, 4>::load(&sqk[buf][t][0][64 * j + 4 * p], qq[j]);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    s[j][e] *= gb.x;
                    if (e % 2) d1 = fmaf(s[j][e], kk[j][e], d1);
                    else d0 = fmaf(s[j][e], kk[j][e], d0);
                }
            }
            const float u = gb.y * (sv[buf][t][cl] - row16_sum(d0 + d1));
            float o0 = 0.f, o1 = 0.f;
#pragma unroll
            for (int j = 0; j < NJ; ++j) {
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    s[j][e] = fmaf(kk[j][e], u, s[j][e]);
                    if (e % 2) o1 = fmaf(s[j][e], qq[j][e], o1);
                    else o0 = fmaf(s[j][e], qq[j][e], o0);
                }
            }
            const float o = row16_sum(o0 + o1);
            if (p == 0) so[t][cl] = o;
        };
        if (nb == TB) {                                         // (a whole batch: no branch between its tokens)
#pragma unroll
            for (int t = 0; t < TB; ++t) token(t);
        } else {
            for (int t = 0; t < nb; ++t) token(t);
        }
        lds_barrier();
        {
            const int t = tid / CW, c = col0 + tid % CW;
            if (t < nb && c < Dv) out[(size_t)(n0 + t) * H * Dv + (size_t)head * Dv + c] = so[t][tid % CW];
        }
        if (more) land(buf ^ 1);
        lds_barrier();
    }
    if (live) {
#pragma unroll
        for (int j = 0; j < NJ; ++j) {
            const int i = 64 * j + 4 * p;
            if (vec && i < D) *reinterpret_cast<float4*>(S + i) = make_float4(s[j][0], s[j][1], s[j][2], s[j][3]);
            else {
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (i + e < D) S[i + e] = s[j][e];
            }
        }
    }
}

SOC_EXPORT int soc_delta_walk(const float* qk, const void* v, const float* gates, int G, int H, int D, int Dv, int Dp, float* state,
                              long long stride, int offset, const int* seq_qstart, const int* seq_rows, float* out, int n_seqs, int dtype,
                              hipStream_t stream) {
    if (n_seqs <= 0) return 0;
    if (G < 1 || H < 1 || H % G || D < 1 || Dv < 1 || Dp != (D + 63) / 64 * 64 || Dp > 256 || n_seqs > 65535 ||
        (D % 4 == 0 && (stride % 4 || offset % 4)))
        return (int)hipErrorInvalidValue;
#define SOC_DW(T, NJ)                                                                                                               \
    hipLaunchKernelGGL((delta_walk_kernel<T, NJ>), dim3(H * ((Dv + 15) / 16), n_seqs), dim3(256), 0, stream, qk, (const T*)v, gates, G, \
                       H, D, Dv, state, (size_t)stride, offset, seq_qstart, seq_rows, out)
#define SOC_DW_T(T) switch (Dp / 64) { case 1: SOC_DW(T, 1); break; case 2: SOC_DW(T, 2); break; case 3: SOC_DW(T, 3); break; default: SOC_DW(T, 4); }
    if (dtype == 0) { SOC_DW_T(float) } else { SOC_DW_T(bf16) }
#undef SOC_DW_T
#undef SOC_DW
    return soc_last_error();
}
