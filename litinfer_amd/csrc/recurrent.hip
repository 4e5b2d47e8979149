// Kernels of recurrent mixers whose state has a fixed size per request: a short causal convolution
// per channel with its tail of past inputs, the selective state-space recurrence
//   S_t = a_t S_{t-1} + dt_t B_t x_t^T,  y_t = S_t^T C_t + D x_t,  a_t = exp(-exp(A_log) dt_t),
// (with `fixed_a`: a_t = fixed_a[head] and dt_t = fixed_dt for every token, a retention with a decay a head; with
// `silu_in` x, B and C pass silu on their way in),
// the gated delta rule, the delta rule with a decay and a removal rate a channel, and the gated RMS norm in groups of columns behind them.  Everything here is float32: inputs, decays,
// step sizes, the state and the sums; only the normed output is rounded to the activations' type.
#include "common.h"

// ------------------------------------------------------------------------------------ causal convolution
// out[t, c] = silu(b[c] + sum_j w[c, j] * u[t - (taps - 1 - j), c]): the last column of w multiplies the
// current token.  Inputs before the first token of the step's portion come from the request's tail
// [slots, taps - 1, C] (its last taps - 1 inputs, zeros for a new request).
__global__ __launch_bounds__(256) void causal_conv_silu_kernel(
    const float* __restrict__ u, long u_stride, int C, int taps, const float* __restrict__ w, const float* __restrict__ b,
    const float* __restrict__ tail, const int* __restrict__ seg_of_token, const int* __restrict__ q_start,
    const int* __restrict__ slots, float* __restrict__ out, long out_stride, float* __restrict__ tail_out) {
    const int t = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
    if (c >= C) return;
    const int seg = seg_of_token[t], i = t - q_start[seg], slot = slots[seg];
    float acc = b ? b[c] : 0.f;
    for (int j = 0; j < taps; ++j) {
        const int back = taps - 1 - j, li = i - back;
        const float v = li >= 0 ? u[(size_t)(t - back) * u_stride + c]
                                : tail[((size_t)slot * (taps - 1) + (taps - 1 + li)) * C + c];
        acc = fmaf(w[(size_t)c * taps + j], v, acc);
        // every request brings one token (tail_out is given then): the thread owns the request's channel and moves
        // its tail up by one as it goes (it has read place j, and will read place j + 1 next)
        if (tail_out && j > 0) tail_out[((size_t)slot * (taps - 1) + (j - 1)) * C + c] = v;
    }
    out[(size_t)t * out_stride + c] = acc / (1.0f + expf(-acc));
}

// The same for many tokens with four neighbouring channels a thread (channels, strides and addresses in multiples of
// four floats): 16-byte loads and stores; the taps' weights of the four channels lie one after the other.
template <int TAPS>
__global__ __launch_bounds__(256) void causal_conv_silu_vec_kernel(
    const float* __restrict__ u, long u_stride, int C, const float* __restrict__ w, const float* __restrict__ b,
    const float* __restrict__ tail, const int* __restrict__ seg_of_token, const int* __restrict__ q_start,
    const int* __restrict__ slots, float* __restrict__ out, long out_stride) {
    const int t = blockIdx.x, c = 4 * (blockIdx.y * 256 + threadIdx.x);
    if (c >= C) return;
    const int seg = seg_of_token[t], i = t - q_start[seg], slot = slots[seg];
    float4 acc = b ? *reinterpret_cast<const float4*>(b + c) : float4{0.f, 0.f, 0.f, 0.f};
    float wv[4][TAPS];
#pragma unroll
    for (int k = 0; k < 4; ++k)
#pragma unroll
        for (int j = 0; j < TAPS; ++j) wv[k][j] = w[(size_t)(c + k) * TAPS + j];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
        const int back = TAPS - 1 - j, li = i - back;
        const float4 v = *reinterpret_cast<const float4*>(li >= 0 ? u + (size_t)(t - back) * u_stride + c
                                                                  : tail + ((size_t)slot * (TAPS - 1) + (TAPS - 1 + li)) * C + c);
        acc.x = fmaf(wv[0][j], v.x, acc.x);
        acc.y = fmaf(wv[1][j], v.y, acc.y);
        acc.z = fmaf(wv[2][j], v.z, acc.z);
        acc.w = fmaf(wv[3][j], v.w, acc.w);
    }
    *reinterpret_cast<float4*>(out + (size_t)t * out_stride + c) =
        float4{acc.x / (1.0f + expf(-acc.x)), acc.y / (1.0f + expf(-acc.y)), acc.z / (1.0f + expf(-acc.z)), acc.w / (1.0f + expf(-acc.w))};
}

// The tail after the step: the last taps - 1 inputs of the request, those of this portion and, where it is
// shorter than that, what is left of the old tail.  A thread owns a (request, channel) and goes upwards, so
// it never reads what it has written.
__global__ __launch_bounds__(256) void conv_tail_update_kernel(
    const float* __restrict__ u, long u_stride, int C, int taps, float* __restrict__ tail,
    const int* __restrict__ q_start, const int* __restrict__ q_len, const int* __restrict__ slots) {
    const int seg = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
    if (c >= C) return;
    const int L = q_len[seg], t0 = q_start[seg];
    float* mine = tail + (size_t)slots[seg] * (taps - 1) * C + c;
    for (int r = 0; r < taps - 1; ++r) {
        const int li = L - (taps - 1) + r;
        mine[(size_t)r * C] = li >= 0 ? u[(size_t)(t0 + li) * u_stride + c] : mine[(size_t)(r + L) * C];
    }
}

extern "C" int li_causal_conv_silu(const float* u, long u_stride, int C, int taps, const float* w, const float* b, float* tail,
                                   const int* seg_of_token, const int* q_start, const int* q_len, const int* slots,
                                   float* out, long out_stride, int T, int segs, int max_q_len, hipStream_t stream) {
    if (T <= 0 || segs <= 0 || C <= 0 || taps <= 0 || taps > 64 || u_stride < C || out_stride < C || max_q_len <= 0) return LI_ERR_SIZE;
    const dim3 grid(T, (C + 255) / 256);
    const bool single = max_q_len == 1 && taps > 1;            // a decoding step: one kernel does both
    const bool vec = !single && T >= 64 && taps >= 2 && taps <= 4 && C % 4 == 0 && u_stride % 4 == 0 && out_stride % 4 == 0 &&
                     ((uintptr_t)u | (uintptr_t)out | (uintptr_t)tail | (uintptr_t)b) % 16 == 0;
    const dim3 grid4(T, (C / 4 + 255) / 256);
    if (vec && taps == 2)
        causal_conv_silu_vec_kernel<2><<<grid4, 256, 0, stream>>>(u, u_stride, C, w, b, tail, seg_of_token, q_start, slots, out, out_stride);
    else if (vec && taps == 3)
        causal_conv_silu_vec_kernel<3><<<grid4, 256, 0, stream>>>(u, u_stride, C, w, b, tail, seg_of_token, q_start, slots, out, out_stride);
    else if (vec)
        causal_conv_silu_vec_kernel<4><<<grid4, 256, 0, stream>>>(u, u_stride, C, w, b, tail, seg_of_token, q_start, slots, out, out_stride);
    else
        causal_conv_silu_kernel<<<grid, 256, 0, stream>>>(u, u_stride, C, taps, w, b, tail, seg_of_token, q_start, slots, out, out_stride,
                                                          single ? tail : nullptr);
    if (taps > 1 && !single) {
        const dim3 g2(segs, (C + 255) / 256);
        conv_tail_update_kernel<<<g2, 256, 0, stream>>>(u, u_stride, C, taps, tail, q_start, q_len, slots);
    }
    return li_launch_status();
}

// ------------------------------------------------------------------------------------ state-space recurrence
// A column p of a head's state (its N values) evolves by itself, given x_t[p] and the head's a_t, dt_t, B_t,
// C_t.  A lane owns NR state values of one column in registers: lane = column * NS + slice, the slices of a
// column are NS neighbouring lanes that add their shares of y up.  A wave is 64 / NS columns of one head; the
// four waves of a block are heads (or column ranges) of ONE group and share its B_t and C_t, which lie in LDS
// for SSM_TB tokens at a time beside each wave's x_t, dt_t and a_t.
//
// A step's portion of a request is cut into chunks of Q tokens that run side by side:
//   MODE 1: the state that a chunk alone builds up from zero, and the product of its decays;
//   the carry kernel: the state with which every chunk begins, chunk after chunk;
//   MODE 0: the recurrence itself from that state, with the outputs; the last chunk leaves the request's state.
// A portion of at most Q tokens (a decoding step) is MODE 0 alone, from the request's state.
#define SSM_TB 16
#define SSM_WAVES 4

__device__ __forceinline__ float silu_f32(float z) { return z / (1.0f + expf(-z)); }
template <bool ON> __device__ __forceinline__ float silu_if(float z) { if constexpr (ON) return silu_f32(z); return z; }
__device__ __forceinline__ float softplus_f32(float z) { return z > 20.f ? z : log1pf(expf(z)); }

template <int NR, int NS, int MODE, bool SILU>
__global__ __launch_bounds__(64 * SSM_WAVES) void ssm_scan_kernel(
    const float* __restrict__ xbc, long xbc_stride, const float* __restrict__ dt_raw, long dt_stride,
    const float* __restrict__ dt_bias, const float* __restrict__ A_log, const float* __restrict__ Dw,
    float* __restrict__ state, const int* __restrict__ slots, const int* __restrict__ q_start, const int* __restrict__ q_len,
    const int* __restrict__ chunk_seg, const int* __restrict__ chunk_idx, float* __restrict__ carry, float* __restrict__ decay,
    float* __restrict__ y, long y_stride, int heads, int vdim, int N, int G, int Q, const float* __restrict__ fixed_a, float fixed_dt) {
    constexpr int NP = NR * NS, PW = 64 / NS;
    extern __shared__ __align__(16) float lds[];
    float* sB = lds;                                   // [SSM_TB][NP]
    float* sC = sB + SSM_TB * NP;                      // [SSM_TB][NP]
    float* sX = sC + SSM_TB * NP;                      // [SSM_WAVES][SSM_TB][PW]
    float* sDt = sX + SSM_WAVES * SSM_TB * PW;         // [SSM_WAVES][SSM_TB]
    float* sA = sDt + SSM_WAVES * SSM_TB;              // [SSM_WAVES][SSM_TB]
    const int bx = blockIdx.x;
    const int seg = chunk_seg ? chunk_seg[bx] : bx;
    if (seg < 0) return;
    const int c = chunk_seg ? chunk_idx[bx] : 0;
    const int L = q_len[seg], first = c * Q;
    if (first >= L) return;
    const int ntok = (L - first < Q) ? L - first : Q;
    const bool last = first + ntok >= L;
    if (MODE == 1 && last) return;                      // nobody needs the last chunk's own state
    const int t0 = q_start[seg] + first;
    const int hpg = heads / G, PS = (vdim + PW - 1) / PW, U = hpg * PS, ublocks = (U + SSM_WAVES - 1) / SSM_WAVES;
    const int g = blockIdx.y / ublocks, ub = blockIdx.y % ublocks;
    const int w = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int unit = ub * SSM_WAVES + w;
    const bool active = unit < U;
    const int head = g * hpg + (active ? unit / PS : 0), pbase = active ? (unit % PS) * PW : 0;
    const int pl = lane / NS, s = lane % NS, p = pbase + pl;
    const int inner = heads * vdim;
    const size_t hoff = (size_t)head * N * vdim;
    float S[NR];
    if (MODE == 0 && active) {
        const float* src = chunk_seg ? carry + (size_t)bx * heads * N * vdim + hoff
                                     : state + (size_t)slots[seg] * heads * N * vdim + hoff;
#pragma unroll
        for (int r = 0; r < NR; ++r) {
            const int n = s * NR + r;
            S[r] = (n < N && p < vdim) ? src[(size_t)n * vdim + p] : 0.f;
        }
    } else {
#pragma unroll
        for (int r = 0; r < NR; ++r) S[r] = 0.f;
    }
    float prod = 1.f;
    const float Dh = (MODE == 0 && active && Dw) ? Dw[head] : 0.f;
    for (int b0 = 0; b0 < ntok; b0 += SSM_TB) {
        __syncthreads();
        for (int i = threadIdx.x; i < SSM_TB * NP; i += 64 * SSM_WAVES) {
            const int tt = i / NP, n = i % NP;
            const bool ok = b0 + tt < ntok && n < N;
            const float* row = xbc + (size_t)(t0 + b0 + tt) * xbc_stride + inner + (size_t)g * N + n;
            sB[i] = ok ? silu_if<SILU>(row[0]) : 0.f;
            sC[i] = ok ? silu_if<SILU>(row[(size_t)G * N]) : 0.f;
        }
        if (active) {
            for (int i = lane; i < SSM_TB * PW; i += 64) {
                const int tt = i / PW, pp = pbase + i % PW;
                const bool ok = b0 + tt < ntok && pp < vdim;
                sX[(w * SSM_TB + tt) * PW + i % PW] = ok ? silu_if<SILU>(xbc[(size_t)(t0 + b0 + tt) * xbc_stride + (size_t)head * vdim + pp]) : 0.f;
            }
            if (lane < SSM_TB) {
                const bool ok = b0 + lane < ntok;
                // (a retention: the same decay and the same step for every token)
                const float d = !ok ? 0.f : fixed_a ? fixed_dt : softplus_f32(dt_raw[(size_t)(t0 + b0 + lane) * dt_stride + head] + dt_bias[head]);
                sDt[w * SSM_TB + lane] = d;
                sA[w * SSM_TB + lane] = fixed_a ? fixed_a[head] : expf(-expf(A_log[head]) * d);
            }
        }
        __syncthreads();
        if (!active) continue;
        const int nt = (ntok - b0 < SSM_TB) ? ntok - b0 : SSM_TB;
        for (int tt = 0; tt < nt; ++tt) {
            const float a = sA[w * SSM_TB + tt], dtv = sDt[w * SSM_TB + tt];
            const float xv = sX[(w * SSM_TB + tt) * PW + pl];
            const float dx = dtv * xv;
            const float4* Bp = reinterpret_cast<const float4*>(sB + tt * NP + s * NR);
            const float4* Cp = reinterpret_cast<const float4*>(sC + tt * NP + s * NR);
            float y0 = 0.f, y1 = 0.f, y2 = 0.f, y3 = 0.f;
#pragma unroll
            for (int r4 = 0; r4 < NR / 4; ++r4) {
                const float4 bv = Bp[r4];
                S[4 * r4 + 0] = fmaf(a, S[4 * r4 + 0], bv.x * dx);
                S[4 * r4 + 1] = fmaf(a, S[4 * r4 + 1], bv.y * dx);
                S[4 * r4 + 2] = fmaf(a, S[4 * r4 + 2], bv.z * dx);
                S[4 * r4 + 3] = fmaf(a, S[4 * r4 + 3], bv.w * dx);
                if (MODE == 0) {
                    const float4 cv = Cp[r4];
                    y0 = fmaf(S[4 * r4 + 0], cv.x, y0);
                    y1 = fmaf(S[4 * r4 + 1], cv.y, y1);
                    y2 = fmaf(S[4 * r4 + 2], cv.z, y2);
                    y3 = fmaf(S[4 * r4 + 3], cv.w, y3);
                }
            }
            if (MODE == 0) {
                float yv = (y0 + y1) + (y2 + y3);
#pragma unroll
                for (int o = 1; o < NS; o <<= 1) yv += __shfl_xor(yv, o, LI_WAVE);
                if (s == 0 && p < vdim) y[(size_t)(t0 + b0 + tt) * y_stride + (size_t)head * vdim + p] = fmaf(Dh, xv, yv);
            } else {
                prod *= a;
            }
        }
    }
    if (!active) return;
    float* dst = nullptr;
    if (MODE == 1) {
        dst = carry + (size_t)bx * heads * N * vdim + hoff;
        if (lane == 0 && pbase == 0) decay[(size_t)bx * heads + head] = prod;
    } else if (last) {
        dst = state + (size_t)slots[seg] * heads * N * vdim + hoff;
    }
    if (dst) {
#pragma unroll
        for (int r = 0; r < NR; ++r) {
            const int n = s * NR + r;
            if (n < N && p < vdim) dst[(size_t)n * vdim + p] = S[r];
        }
    }
}

// The same recurrence with FOUR neighbouring columns a lane (head sizes that are multiples of 4): lane = quad * NS +
// slice holds NR state values of each of its four columns.  A value of B_t or C_t read from LDS then serves four
// state elements instead of one, and the state comes from and goes to memory in 16-byte pieces.  A wave is 256 / NS
// columns of one head.  Modes, chunks and blocks as above.
template <int NR, int NS, int MODE, bool SILU>
__global__ __launch_bounds__(64 * SSM_WAVES) void ssm_scan_quad_kernel(
    const float* __restrict__ xbc, long xbc_stride, const float* __restrict__ dt_raw, long dt_stride,
    const float* __restrict__ dt_bias, const float* __restrict__ A_log, const float* __restrict__ Dw,
    float* __restrict__ state, const int* __restrict__ slots, const int* __restrict__ q_start, const int* __restrict__ q_len,
    const int* __restrict__ chunk_seg, const int* __restrict__ chunk_idx, float* __restrict__ carry, float* __restrict__ decay,
    float* __restrict__ y, long y_stride, int heads, int vdim, int N, int G, int Q, const float* __restrict__ fixed_a, float fixed_dt) {
    constexpr int NP = NR * NS, PW = 256 / NS;
    extern __shared__ __align__(16) float lds[];
    float* sB = lds;                                   // [SSM_TB][NP]
    float* sC = sB + SSM_TB * NP;                      // [SSM_TB][NP]
    float* sX = sC + SSM_TB * NP;                      // [SSM_WAVES][SSM_TB][PW]
    float* sDt = sX + SSM_WAVES * SSM_TB * PW;         // [SSM_WAVES][SSM_TB]
    float* sA = sDt + SSM_WAVES * SSM_TB;              // [SSM_WAVES][SSM_TB]
    const int bx = blockIdx.x;
    const int seg = chunk_seg ? chunk_seg[bx] : bx;
    if (seg < 0) return;
    const int c = chunk_seg ? chunk_idx[bx] : 0;
    const int L = q_len[seg], first = c * Q;
    if (first >= L) return;
    const int ntok = (L - first < Q) ? L - first : Q;
    const bool last = first + ntok >= L;
    if (MODE == 1 && last) return;
    const int t0 = q_start[seg] + first;
    const int hpg = heads / G, PS = (vdim + PW - 1) / PW, U = hpg * PS, ublocks = (U + SSM_WAVES - 1) / SSM_WAVES;
    const int g = blockIdx.y / ublocks, ub = blockIdx.y % ublocks;
    const int w = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int unit = ub * SSM_WAVES + w;
    const bool active = unit < U;
    const int head = g * hpg + (active ? unit / PS : 0), pbase = active ? (unit % PS) * PW : 0;
    const int pq = lane / NS, s = lane % NS, p = pbase + 4 * pq;        // the first of the lane's four columns
    const bool cols = p < vdim;                                         // (vdim is a multiple of 4: all four or none)
    const int inner = heads * vdim;
    const size_t hoff = (size_t)head * N * vdim;
    float4 S[NR];
    if (MODE == 0 && active) {
        const float* src = chunk_seg ? carry + (size_t)bx * heads * N * vdim + hoff
                                     : state + (size_t)slots[seg] * heads * N * vdim + hoff;
#pragma unroll
        for (int r = 0; r < NR; ++r) {
            const int n = s * NR + r;
            S[r] = (n < N && cols) ? *reinterpret_cast<const float4*>(src + (size_t)n * vdim + p) : float4{0.f, 0.f, 0.f, 0.f};
        }
    } else {
#pragma unroll
        for (int r = 0; r < NR; ++r) S[r] = float4{0.f, 0.f, 0.f, 0.f};
    }
    float prod = 1.f;
    const float Dh = (MODE == 0 && active && Dw) ? Dw[head] : 0.f;
    for (int b0 = 0; b0 < ntok; b0 += SSM_TB) {
        __syncthreads();
        for (int i = threadIdx.x; i < SSM_TB * NP; i += 64 * SSM_WAVES) {
            const int tt = i / NP, n = i % NP;
            const bool ok = b0 + tt < ntok && n < N;
            const float* row = xbc + (size_t)(t0 + b0 + tt) * xbc_stride + inner + (size_t)g * N + n;
            sB[i] = ok ? silu_if<SILU>(row[0]) : 0.f;
            sC[i] = ok ? silu_if<SILU>(row[(size_t)G * N]) : 0.f;
        }
        if (active) {
            for (int i = lane; i < SSM_TB * PW; i += 64) {
                const int tt = i / PW, pp = pbase + i % PW;
                const bool ok = b0 + tt < ntok && pp < vdim;
                sX[(w * SSM_TB + tt) * PW + i % PW] = ok ? silu_if<SILU>(xbc[(size_t)(t0 + b0 + tt) * xbc_stride + (size_t)head * vdim + pp]) : 0.f;
            }
            if (lane < SSM_TB) {
                const bool ok = b0 + lane < ntok;
                // (a retention: the same decay and the same step for every token)
                const float d = !ok ? 0.f : fixed_a ? fixed_dt : softplus_f32(dt_raw[(size_t)(t0 + b0 + lane) * dt_stride + head] + dt_bias[head]);
                sDt[w * SSM_TB + lane] = d;
                sA[w * SSM_TB + lane] = fixed_a ? fixed_a[head] : expf(-expf(A_log[head]) * d);
            }
        }
        __syncthreads();
        if (!active) continue;
        const int nt = (ntok - b0 < SSM_TB) ? ntok - b0 : SSM_TB;
        for (int tt = 0; tt < nt; ++tt) {
            const float a = sA[w * SSM_TB + tt], dtv = sDt[w * SSM_TB + tt];
            const float4 xv = *reinterpret_cast<const float4*>(sX + (w * SSM_TB + tt) * PW + 4 * pq);
            const float4 dx = float4{dtv * xv.x, dtv * xv.y, dtv * xv.z, dtv * xv.w};
            const float4* Bp = reinterpret_cast<const float4*>(sB + tt * NP + s * NR);
            const float4* Cp = reinterpret_cast<const float4*>(sC + tt * NP + s * NR);
            float4 yv = float4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int r4 = 0; r4 < NR / 4; ++r4) {
                const float4 bv = Bp[r4];
                const float bs[4] = {bv.x, bv.y, bv.z, bv.w};
                float cs[4] = {0.f, 0.f, 0.f, 0.f};
                if (MODE == 0) { const float4 cv = Cp[r4]; cs[0] = cv.x; cs[1] = cv.y; cs[2] = cv.z; cs[3] = cv.w; }
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    float4& st = S[4 * r4 + j];
                    st.x = fmaf(a, st.x, bs[j] * dx.x);
                    st.y = fmaf(a, st.y, bs[j] * dx.y);
                    st.z = fmaf(a, st.z, bs[j] * dx.z);
                    st.w = fmaf(a, st.w, bs[j] * dx.w);
                    if (MODE == 0) {
                        yv.x = fmaf(st.x, cs[j], yv.x);
                        yv.y = fmaf(st.y, cs[j], yv.y);
                        yv.z = fmaf(st.z, cs[j], yv.z);
                        yv.w = fmaf(st.w, cs[j], yv.w);
                    }
                }
            }
            if (MODE == 0) {
#pragma unroll
                for (int o = 1; o < NS; o <<= 1) {
                    yv.x += __shfl_xor(yv.x, o, LI_WAVE);
                    yv.y += __shfl_xor(yv.y, o, LI_WAVE);
                    yv.z += __shfl_xor(yv.z, o, LI_WAVE);
                    yv.w += __shfl_xor(yv.w, o, LI_WAVE);
                }
                if (s == 0 && cols)
                    *reinterpret_cast<float4*>(y + (size_t)(t0 + b0 + tt) * y_stride + (size_t)head * vdim + p) =
                        float4{fmaf(Dh, xv.x, yv.x), fmaf(Dh, xv.y, yv.y), fmaf(Dh, xv.z, yv.z), fmaf(Dh, xv.w, yv.w)};
            } else {
                prod *= a;
            }
        }
    }
    if (!active) return;
    float* dst = nullptr;
    if (MODE == 1) {
        dst = carry + (size_t)bx * heads * N * vdim + hoff;
        if (lane == 0 && pbase == 0) decay[(size_t)bx * heads + head] = prod;
    } else if (last) {
        dst = state + (size_t)slots[seg] * heads * N * vdim + hoff;
    }
    if (dst && cols) {
#pragma unroll
        for (int r = 0; r < NR; ++r) {
            const int n = s * NR + r;
            if (n < N) *reinterpret_cast<float4*>(dst + (size_t)n * vdim + p) = S[r];
        }
    }
}

// Numbers the chunks of a step: request after request, chunk after chunk.  chunk_first[seg] is a request's
// first chunk; chunk_seg / chunk_idx say whose chunk, and which of its chunks, a number is (-1: none).
__global__ __launch_bounds__(256) void ssm_chunk_index_kernel(const int* __restrict__ q_len, int segs, int Q, int max_chunks,
                                                              int* __restrict__ chunk_seg, int* __restrict__ chunk_idx,
                                                              int* __restrict__ chunk_first) {
    if (threadIdx.x == 0) {
        int at = 0;
        for (int sgm = 0; sgm < segs; ++sgm) {
            chunk_first[sgm] = at;
            at += (q_len[sgm] + Q - 1) / Q;
        }
        chunk_first[segs] = at;
    }
    for (int i = threadIdx.x; i < max_chunks; i += 256) chunk_seg[i] = -1;
    __syncthreads();
    for (int sgm = threadIdx.x; sgm < segs; sgm += 256) {
        const int f = chunk_first[sgm], n = chunk_first[sgm + 1] - f;
        for (int k = 0; k < n && f + k < max_chunks; ++k) { chunk_seg[f + k] = sgm; chunk_idx[f + k] = k; }
    }
}

// carry[chunk] holds what the chunk alone built up from zero; afterwards it holds the state with which the
// chunk begins: the request's state for its first chunk, decay * (state before) + (built up before) onwards.
__global__ __launch_bounds__(256) void ssm_carry_kernel(float* __restrict__ carry, const float* __restrict__ decay,
                                                        const float* __restrict__ state, const int* __restrict__ slots,
                                                        const int* __restrict__ q_len, const int* __restrict__ chunk_first,
                                                        int heads, int NV, int Q) {
    const int seg = blockIdx.x, head = blockIdx.y;
    const int nch = (q_len[seg] + Q - 1) / Q, base = chunk_first[seg];
    const float* st = state + ((size_t)slots[seg] * heads + head) * NV;
    for (int e = blockIdx.z * 256 + threadIdx.x; e < NV; e += gridDim.z * 256) {
        float run = st[e];
        for (int k = 0; k < nch; ++k) {
            float* at = carry + ((size_t)(base + k) * heads + head) * NV + e;
            float next = 0.f;
            if (k + 1 < nch) next = fmaf(decay[(size_t)(base + k) * heads + head], run, *at);
            *at = run;
            run = next;
        }
    }
}

template <int NR, int NS, bool QUAD, bool SILU>
static int ssm_launch_as(const float* xbc, long xbc_stride, const float* dt_raw, long dt_stride, const float* dt_bias,
                      const float* A_log, const float* Dw, float* state, const int* slots, const int* q_start, const int* q_len,
                      int* chunk_tab, float* carry, float* decay, float* y, long y_stride, int heads, int vdim, int N, int G,
                      int Q, int segs, int max_chunks, bool chunked, const float* fixed_a, float fixed_dt, hipStream_t stream) {
    constexpr int NP = NR * NS, PW = (QUAD ? 256 : 64) / NS;
    const size_t lds = (size_t)(2 * SSM_TB * NP + SSM_WAVES * SSM_TB * PW + 2 * SSM_WAVES * SSM_TB) * sizeof(float);
#define SSM_KERNEL(MODE_) (QUAD ? ssm_scan_quad_kernel<(QUAD ? NR : 4), (QUAD ? NS : 2), MODE_, SILU> : ssm_scan_kernel<(QUAD ? 16 : NR), (QUAD ? 1 : NS), MODE_, SILU>)
    const int hpg = heads / G, PS = (vdim + PW - 1) / PW, U = hpg * PS, ublocks = (U + SSM_WAVES - 1) / SSM_WAVES;
    if (!chunked) {
        const dim3 grid(segs, G * ublocks);
        SSM_KERNEL(0)<<<grid, 64 * SSM_WAVES, lds, stream>>>(xbc, xbc_stride, dt_raw, dt_stride, dt_bias, A_log, Dw,
            state, slots, q_start, q_len, nullptr, nullptr, nullptr, nullptr, y, y_stride, heads, vdim, N, G, Q, fixed_a, fixed_dt);
        return li_launch_status();
    }
    int* chunk_seg = chunk_tab;
    int* chunk_idx = chunk_tab + max_chunks;
    int* chunk_first = chunk_tab + 2 * max_chunks;
    ssm_chunk_index_kernel<<<1, 256, 0, stream>>>(q_len, segs, Q, max_chunks, chunk_seg, chunk_idx, chunk_first);
    const dim3 grid(max_chunks, G * ublocks);
    SSM_KERNEL(1)<<<grid, 64 * SSM_WAVES, lds, stream>>>(xbc, xbc_stride, dt_raw, dt_stride, dt_bias, A_log, Dw,
        state, slots, q_start, q_len, chunk_seg, chunk_idx, carry, decay, y, y_stride, heads, vdim, N, G, Q, fixed_a, fixed_dt);
    const int NV = N * vdim;
    int zs = (NV + 255) / 256;
    if (zs > 16) zs = 16;
    ssm_carry_kernel<<<dim3(segs, heads, zs), 256, 0, stream>>>(carry, decay, state, slots, q_len, chunk_first, heads, NV, Q);
    SSM_KERNEL(0)<<<grid, 64 * SSM_WAVES, lds, stream>>>(xbc, xbc_stride, dt_raw, dt_stride, dt_bias, A_log, Dw,
        state, slots, q_start, q_len, chunk_seg, chunk_idx, carry, decay, y, y_stride, heads, vdim, N, G, Q, fixed_a, fixed_dt);
    return li_launch_status();
#undef SSM_KERNEL
}

template <int NR, int NS, bool QUAD, typename... A>
static int ssm_launch(int silu_in, A... args) { return silu_in ? ssm_launch_as<NR, NS, QUAD, true>(args...) : ssm_launch_as<NR, NS, QUAD, false>(args...); }

// ------------------------------------------------------------------------------- retention of long portions, as products
// With the same decay a for every token of a head the recurrence S_t = a S_(t-1) + f k_t v_t^T, y_t = S_t^T q_t over a chunk
// of n <= 64 tokens (numbered from 0) that begins with the state S is
//     y_i = a^(i+1) q_i S + sum_(j<=i) a^(i-j) f (q_i . k_j) v_j,      S' = a^n S + sum_j a^(n-1-j) f k_j v_j^T,
// three matrix products, on the float32 matrix cores (v_mfma_f32_32x32x2_f32: float32 operands, products and sums; lane l of
// the row operand holds row l % 32 and k-value l / 32, of the column operand column l % 32 and k-value l / 32, of the result
// column l % 32 and, in register r, row 8 (r / 4) + 4 (l / 32) + r % 4).  A decay is only ever raised to powers >= 0.
//   retention_states_kernel: the second term of S' of every chunk;
//   retention_carry_kernel: the state with which every chunk begins, chunk after chunk, and the request's state at the end;
//   retention_outputs_kernel: the outputs.
// Which k-value a step of the matrix cores takes is free as long as both operands agree: the scores K Q^T take the four
// k-values 8 t + 4 (l / 32) .. + 3 of a 16-byte piece in four steps, and their result, keys as rows, is the row operand of
// the product with V as it is (register r holds the key whose number the column operand then reads).
#define RET_Q 64               // tokens of a chunk (SSM chunks of the same length are what the host numbers)
typedef float ret_f32x16 __attribute__((ext_vector_type(16)));

__device__ __forceinline__ float4 silu_if4(float4 v, int on) { return on ? float4{silu_f32(v.x), silu_f32(v.y), silu_f32(v.z), silu_f32(v.w)} : v; }

// WT: fragments of 32 rows (state values) and of 32 columns a wave; the four waves are two by two, a block takes 64 WT of both.
template <int WT>
__global__ __launch_bounds__(256) void retention_states_kernel(
    const float* __restrict__ xbc, long xbc_stride, const int* __restrict__ q_start, const int* __restrict__ q_len,
    const int* __restrict__ chunk_seg, const int* __restrict__ chunk_idx, float* __restrict__ carry, int heads, int vdim, int N,
    const float* __restrict__ fixed_a, float step, int silu_in) {
    constexpr int B = 64 * WT;
    extern __shared__ __align__(16) float lds[];
    float* sK = lds;                                   // [RET_Q][B]
    float* sV = lds + RET_Q * B;                       // [RET_Q][B], times a^(n-1-j) f
    const int bx = blockIdx.x, seg = chunk_seg[bx];
    if (seg < 0) return;
    const int first = chunk_idx[bx] * RET_Q, L = q_len[seg];
    const int ntok = L - first < RET_Q ? L - first : RET_Q, t0 = q_start[seg] + first, head = blockIdx.y;
    const int vb = (vdim + B - 1) / B, n0 = (blockIdx.z / vb) * B, p0 = (blockIdx.z % vb) * B;
    const float a = fixed_a[head];
    const int inner = heads * vdim;
    const int rows = (ntok + 1) & ~1;                  // (whole pairs of tokens: the row behind an odd last one is zero)
    for (int i = threadIdx.x; i < rows * (B / 4); i += 256) {
        const int j = i / (B / 4), c = 4 * (i % (B / 4));
        const float* row = xbc + (size_t)(t0 + j) * xbc_stride;
        float4 k = float4{0.f, 0.f, 0.f, 0.f}, v = k;
        if (j < ntok && n0 + c < N) k = silu_if4(*reinterpret_cast<const float4*>(row + inner + (size_t)head * N + n0 + c), silu_in);
        if (j < ntok && p0 + c < vdim) {
            v = silu_if4(*reinterpret_cast<const float4*>(row + (size_t)head * vdim + p0 + c), silu_in);
            const float f = powf(a, (float)(ntok - 1 - j)) * step;
            v = float4{v.x * f, v.y * f, v.z * f, v.w * f};
        }
        *reinterpret_cast<float4*>(sK + j * B + c) = k;
        *reinterpret_cast<float4*>(sV + j * B + c) = v;
    }
    __syncthreads();
    const int w = threadIdx.x >> 6, lane = threadIdx.x & 63, ql = lane & 31, h = lane >> 5;
    const int wn = (w >> 1) * 32 * WT, wp = (w & 1) * 32 * WT;
    if (n0 + wn >= N || p0 + wp >= vdim) return;
    ret_f32x16 acc[WT][WT];
#pragma unroll
    for (int x = 0; x < WT; ++x)
#pragma unroll
        for (int y = 0; y < WT; ++y)
#pragma unroll
            for (int r = 0; r < 16; ++r) acc[x][y][r] = 0.f;
#pragma unroll 4
    for (int j = 0; j < rows; j += 2) {
        float kf[WT], vf[WT];
#pragma unroll
        for (int x = 0; x < WT; ++x) { kf[x] = sK[(j + h) * B + wn + 32 * x + ql]; vf[x] = sV[(j + h) * B + wp + 32 * x + ql]; }
#pragma unroll
        for (int x = 0; x < WT; ++x)
#pragma unroll
            for (int y = 0; y < WT; ++y) acc[x][y] = __builtin_amdgcn_mfma_f32_32x32x2f32(kf[x], vf[y], acc[x][y], 0, 0, 0);
    }
    float* dst = carry + ((size_t)bx * heads + head) * N * vdim;
#pragma unroll
    for (int x = 0; x < WT; ++x)
#pragma unroll
        for (int y = 0; y < WT; ++y)
#pragma unroll
            for (int r = 0; r < 16; ++r) {
                const int n = n0 + wn + 32 * x + 8 * (r >> 2) + 4 * h + (r & 3), p = p0 + wp + 32 * y + ql;
                if (n < N && p < vdim) dst[(size_t)n * vdim + p] = acc[x][y][r];
            }
}

// carry[chunk]: in: what the chunk alone adds; out: the state with which it begins.  The next eight chunks' values are on
// their way while a chunk is worked on.  NV4: a head's state in 16-byte pieces.
#define RET_AHEAD 8
__global__ __launch_bounds__(64) void retention_carry_kernel(float4* __restrict__ carry, float4* __restrict__ state,
                                                             const int* __restrict__ slots, const int* __restrict__ q_len,
                                                             const int* __restrict__ chunk_first, int heads, int NV4,
                                                             const float* __restrict__ fixed_a) {
    const int seg = blockIdx.x, head = blockIdx.y, e = blockIdx.z * 64 + threadIdx.x;
    if (e >= NV4) return;
    const int L = q_len[seg], nch = (L + RET_Q - 1) / RET_Q;
    const float a = fixed_a[head], whole = powf(a, (float)RET_Q), tail = powf(a, (float)(L - (nch - 1) * RET_Q));
    float4* at = carry + ((size_t)chunk_first[seg] * heads + head) * NV4 + e;
    const size_t next = (size_t)heads * NV4;
    float4* st = state + ((size_t)slots[seg] * heads + head) * NV4 + e;
    float4 run = *st, own[RET_AHEAD];
#pragma unroll
    for (int u = 0; u < RET_AHEAD; ++u) own[u] = at[(size_t)(u < nch ? u : nch - 1) * next];
    for (int c0 = 0; c0 < nch; c0 += RET_AHEAD) {
        float4 ahead[RET_AHEAD];
#pragma unroll
        for (int u = 0; u < RET_AHEAD; ++u) {
            const int c = c0 + RET_AHEAD + u;
            ahead[u] = at[(size_t)(c < nch ? c : nch - 1) * next];      // (past the end: the last chunk's again, not used)
        }
#pragma unroll
        for (int u = 0; u < RET_AHEAD; ++u) {
            const int c = c0 + u;
            if (c < nch) {
                const float f = c + 1 < nch ? whole : tail;
                at[(size_t)c * next] = run;
                run = float4{fmaf(f, run.x, own[u].x), fmaf(f, run.y, own[u].y), fmaf(f, run.z, own[u].z), fmaf(f, run.w, own[u].w)};
            }
        }
#pragma unroll
        for (int u = 0; u < RET_AHEAD; ++u) own[u] = ahead[u];
    }
    *st = run;
}

// NQ: 8-value pieces of a query (N <= 8 NQ); PT: fragments of 32 columns a wave.  The four waves are two query tiles of 32 by two
// column ranges; a query lies in registers (16-byte pieces 2 t + l / 32 of row l % 32), keys and values in LDS.
template <int NQ, int PT>
__global__ __launch_bounds__(256) void retention_outputs_kernel(
    const float* __restrict__ xbc, long xbc_stride, const int* __restrict__ q_start, const int* __restrict__ q_len,
    const int* __restrict__ chunk_seg, const int* __restrict__ chunk_idx, const float* __restrict__ carry, float* __restrict__ y,
    long y_stride, int heads, int vdim, int N, const float* __restrict__ fixed_a, float step, int silu_in) {
    constexpr int NP = 8 * NQ, KS = NP + 4, VB = 64 * PT;
    extern __shared__ __align__(16) float lds[];
    float* sK = lds;                                   // [RET_Q][KS]: four floats of padding spread the 16-byte reads over the banks
    float* sV = sK + RET_Q * KS;                       // [RET_Q][VB]
    float* pw = sV + RET_Q * VB;                       // [RET_Q + 1]: the powers of the decay
    const int bx = blockIdx.x, seg = chunk_seg[bx];
    if (seg < 0) return;
    const int first = chunk_idx[bx] * RET_Q, L = q_len[seg];
    const int ntok = L - first < RET_Q ? L - first : RET_Q, t0 = q_start[seg] + first, head = blockIdx.y, p0 = blockIdx.z * VB;
    const int inner = heads * vdim;
    const int w = threadIdx.x >> 6, lane = threadIdx.x & 63, ql = lane & 31, h = lane >> 5;
    const int it = w >> 1, pc = p0 + (w & 1) * 32 * PT, i = it * 32 + ql;
    // the wave's queries, asked for before keys and values are staged
    float4 q[NQ];
    {
        const float* row = xbc + (size_t)(t0 + (i < ntok ? i : ntok - 1)) * xbc_stride + inner + (size_t)(heads + head) * N;
#pragma unroll
        for (int t = 0; t < NQ; ++t) {
            const int n = 8 * t + 4 * h;
            q[t] = n < N ? *reinterpret_cast<const float4*>(row + n) : float4{0.f, 0.f, 0.f, 0.f};
        }
    }
    if (threadIdx.x <= RET_Q) pw[threadIdx.x] = powf(fixed_a[head], (float)threadIdx.x);
    for (int x = threadIdx.x; x < RET_Q * (NP / 4); x += 256) {
        const int j = x / (NP / 4), c = 4 * (x % (NP / 4));
        float4 k = float4{0.f, 0.f, 0.f, 0.f};
        if (j < ntok && c < N) k = silu_if4(*reinterpret_cast<const float4*>(xbc + (size_t)(t0 + j) * xbc_stride + inner + (size_t)head * N + c), silu_in);
        *reinterpret_cast<float4*>(sK + j * KS + c) = k;
    }
    for (int x = threadIdx.x; x < RET_Q * (VB / 4); x += 256) {
        const int j = x / (VB / 4), c = 4 * (x % (VB / 4));
        float4 v = float4{0.f, 0.f, 0.f, 0.f};
        if (j < ntok && p0 + c < vdim) v = silu_if4(*reinterpret_cast<const float4*>(xbc + (size_t)(t0 + j) * xbc_stride + (size_t)head * vdim + p0 + c), silu_in);
        *reinterpret_cast<float4*>(sV + j * VB + c) = v;
    }
#pragma unroll
    for (int t = 0; t < NQ; ++t) q[t] = silu_if4(q[t], silu_in);        // (silu(0) = 0)
    __syncthreads();
    if (it * 32 >= ntok || pc >= vdim) return;
    ret_f32x16 out[PT];
#pragma unroll
    for (int pt = 0; pt < PT; ++pt)
#pragma unroll
        for (int r = 0; r < 16; ++r) out[pt][r] = 0.f;
    for (int jt = 0; jt <= it; ++jt) {
        ret_f32x16 sc;                                 // keys as rows, the wave's queries as columns
#pragma unroll
        for (int r = 0; r < 16; ++r) sc[r] = 0.f;
        const float* krow = sK + (jt * 32 + ql) * KS + 4 * h;
#pragma unroll
        for (int t = 0; t < NQ; ++t) {
            const float4 k = *reinterpret_cast<const float4*>(krow + 8 * t);
            sc = __builtin_amdgcn_mfma_f32_32x32x2f32(k.x, q[t].x, sc, 0, 0, 0);
            sc = __builtin_amdgcn_mfma_f32_32x32x2f32(k.y, q[t].y, sc, 0, 0, 0);
            sc = __builtin_amdgcn_mfma_f32_32x32x2f32(k.z, q[t].z, sc, 0, 0, 0);
            sc = __builtin_amdgcn_mfma_f32_32x32x2f32(k.w, q[t].w, sc, 0, 0, 0);
        }
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            const int d = i - (jt * 32 + 8 * (r >> 2) + 4 * h + (r & 3));
            sc[r] = d >= 0 ? sc[r] * (pw[d >= 0 ? d : 0] * step) : 0.f;
        }
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            const float* vrow = sV + (jt * 32 + 8 * (r >> 2) + 4 * h + (r & 3)) * VB + (pc - p0) + ql;
#pragma unroll
            for (int pt = 0; pt < PT; ++pt) out[pt] = __builtin_amdgcn_mfma_f32_32x32x2f32(sc[r], vrow[32 * pt], out[pt], 0, 0, 0);
        }
    }
    // what the state at the chunk's beginning adds
    const float* S = carry + ((size_t)bx * heads + head) * N * vdim;
    const float f = pw[i + 1];
    int col[PT];
#pragma unroll
    for (int pt = 0; pt < PT; ++pt) col[pt] = pc + 32 * pt + ql < vdim ? pc + 32 * pt + ql : vdim - 1;     // (a column past the last is not written)
#pragma unroll
    for (int t = 0; t < NQ; ++t) {
        const float qs[4] = {q[t].x * f, q[t].y * f, q[t].z * f, q[t].w * f};
        float sv[4][PT];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int n = 8 * t + 4 * h + e;
            const float* row = S + (size_t)(n < N ? n : N - 1) * vdim;          // (a value past the last meets a zero of q)
#pragma unroll
            for (int pt = 0; pt < PT; ++pt) sv[e][pt] = row[col[pt]];
        }
#pragma unroll
        for (int e = 0; e < 4; ++e)
#pragma unroll
            for (int pt = 0; pt < PT; ++pt) out[pt] = __builtin_amdgcn_mfma_f32_32x32x2f32(qs[e], sv[e][pt], out[pt], 0, 0, 0);
    }
#pragma unroll
    for (int pt = 0; pt < PT; ++pt)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            const int row = it * 32 + 8 * (r >> 2) + 4 * h + (r & 3), p = pc + 32 * pt + ql;
            if (row < ntok && p < vdim) y[(size_t)(t0 + row) * y_stride + (size_t)head * vdim + p] = out[pt][r];
        }
}

template <int NQ, int PT>
static int retention_outputs_launch(const dim3& grid, const float* xbc, long xbc_stride, const int* q_start, const int* q_len,
                                    const int* chunk_seg, const int* chunk_idx, const float* carry, float* y, long y_stride,
                                    int heads, int vdim, int N, const float* fixed_a, float step, int silu_in, hipStream_t stream) {
    constexpr int bytes = (RET_Q * (8 * NQ + 4) + RET_Q * 64 * PT + RET_Q + 4) * 4;
    static bool configured = false;
    if (!configured) {
        if (hipFuncSetAttribute((const void*)retention_outputs_kernel<NQ, PT>, hipFuncAttributeMaxDynamicSharedMemorySize, bytes) != hipSuccess)
            return LI_ERR_LAUNCH;
        configured = true;
    }
    retention_outputs_kernel<NQ, PT><<<grid, 256, bytes, stream>>>(xbc, xbc_stride, q_start, q_len, chunk_seg, chunk_idx, carry, y, y_stride,
                                                                   heads, vdim, N, fixed_a, step, silu_in);
    return li_launch_status();
}

// The chunked form of a retention (every head with keys of its own); operands in 16-byte pieces, N and vdim multiples of four.
static int retention_launch(const float* xbc, long xbc_stride, float* state, const int* slots, const int* q_start, const int* q_len,
                            int* chunk_tab, float* carry, float* y, long y_stride, int heads, int vdim, int N, int segs, int max_chunks,
                            const float* fixed_a, float step, int silu_in, hipStream_t stream) {
    int* chunk_seg = chunk_tab;
    int* chunk_idx = chunk_tab + max_chunks;
    int* chunk_first = chunk_tab + 2 * max_chunks;
    ssm_chunk_index_kernel<<<1, 256, 0, stream>>>(q_len, segs, RET_Q, max_chunks, chunk_seg, chunk_idx, chunk_first);
    const int wt = (N > 64 || vdim > 64) ? 2 : 1, b = 64 * wt;
    const dim3 gs(max_chunks, heads, ((N + b - 1) / b) * ((vdim + b - 1) / b));
    if (wt == 2) retention_states_kernel<2><<<gs, 256, 2 * RET_Q * 128 * 4, stream>>>(xbc, xbc_stride, q_start, q_len, chunk_seg, chunk_idx, carry, heads, vdim, N, fixed_a, step, silu_in);
    else retention_states_kernel<1><<<gs, 256, 2 * RET_Q * 64 * 4, stream>>>(xbc, xbc_stride, q_start, q_len, chunk_seg, chunk_idx, carry, heads, vdim, N, fixed_a, step, silu_in);
    const int NV4 = N * vdim / 4;
    retention_carry_kernel<<<dim3(segs, heads, (NV4 + 63) / 64), 64, 0, stream>>>((float4*)carry, (float4*)state, slots, q_len, chunk_first, heads, NV4, fixed_a);
    const int pt = vdim > 64 ? 2 : 1;
    const dim3 go(max_chunks, heads, (vdim + 64 * pt - 1) / (64 * pt));
#define RET_GO(NQ_)                                                                                                                  \
    return pt == 2 ? retention_outputs_launch<NQ_, 2>(go, xbc, xbc_stride, q_start, q_len, chunk_seg, chunk_idx, carry, y, y_stride, heads, vdim, N, fixed_a, step, silu_in, stream) \
                   : retention_outputs_launch<NQ_, 1>(go, xbc, xbc_stride, q_start, q_len, chunk_seg, chunk_idx, carry, y, y_stride, heads, vdim, N, fixed_a, step, silu_in, stream)
    if (N <= 32) RET_GO(4);
    if (N <= 64) RET_GO(8);
    if (N <= 128) RET_GO(16);
    RET_GO(32);
#undef RET_GO
}

// The four-columns-a-lane layout for a state of N values a column and heads of vdim columns (a multiple of 4): lanes
// a quad of columns (2 to 16) and values a lane and column (4 to 32); 0 if it has none.
static int ssm_quad_layout(int N, int vdim, int* slices, int* per_lane) {
    if (N <= 0 || N > 256 || vdim <= 0 || vdim % 4) return 0;
    int ns = 2;
    while (ns < 16 && 256 / (2 * ns) >= vdim) ns *= 2;      // narrow heads: more lanes a quad, so that a wave is full
    while (ns < 16 && (N + ns - 1) / ns > 32) ns *= 2;      // at most 32 values a lane and column (128 registers)
    const int need = (N + ns - 1) / ns;
    const int nr = need <= 4 ? 4 : need <= 8 ? 8 : need <= 16 ? 16 : need <= 32 ? 32 : 0;
    if (!nr || ns * nr > 256) return 0;
    *slices = ns;
    *per_lane = nr;
    return 1;
}

// How a state of N values a column is spread: slices (lanes a column) and values a lane; 0 if no kernel has it.
extern "C" int li_ssm_scan_layout(int N, int vdim, int* slices, int* per_lane) {
    if (N <= 0 || N > 256 || vdim <= 0) return 0;
    int ns = 1;
    while (ns < 4 && 64 / (2 * ns) >= vdim) ns *= 2;        // few columns a head: more lanes a column, so that a wave is full
    while (ns < 4 && (N + ns - 1) / ns > 128) ns *= 2;
    const int need = (N + ns - 1) / ns;
    int nr = need <= 16 ? 16 : need <= 32 ? 32 : need <= 64 ? 64 : need <= 128 ? 128 : 0;
    if (!nr) return 0;
    while (ns * nr > 256 && ns > 1 && (N + ns / 2 - 1) / (ns / 2) <= 128) {     // no more padding than LDS has room for
        ns /= 2;
        const int nd = (N + ns - 1) / ns;
        nr = nd <= 16 ? 16 : nd <= 32 ? 32 : nd <= 64 ? 64 : 128;
    }
    if (ns * nr > 256) return 0;
    if (slices) *slices = ns;
    if (per_lane) *per_lane = nr;
    return 1;
}

// Chunks that a step of T tokens in `segs` portions can have at most, and the bytes of the tables and states
// that the chunked form keeps in the workspace.
extern "C" long li_ssm_scan_work_bytes(int T, int segs, int heads, int vdim, int N, int Q, int* max_chunks) {
    const long mc = (long)T / Q + segs;
    if (max_chunks) *max_chunks = (int)mc;
    const long ints = ((3 * mc + segs + 1 + 3) / 4) * 4;
    return ints * 4 + mc * heads * ((long)N * vdim + 1) * 4;
}

extern "C" int li_ssm_scan(const float* xbc, long xbc_stride, const float* dt_raw, long dt_stride, const float* dt_bias,
                           const float* A_log, const float* Dw, float* state, const int* slots, const int* q_start,
                           const int* q_len, float* y, long y_stride, int heads, int vdim, int N, int G, int Q, int T,
                           int segs, int max_q_len, void* work, long work_bytes, const float* fixed_a, float fixed_dt, int silu_in, hipStream_t stream) {
    if (T <= 0 || segs <= 0 || heads <= 0 || G <= 0 || heads % G || vdim <= 0 || N <= 0 || Q <= 0 || max_q_len <= 0 ||
        xbc_stride < (long)heads * vdim + 2L * G * N || (!fixed_a && (dt_stride < heads || !dt_raw || !dt_bias || !A_log)) || y_stride < (long)heads * vdim)
        return LI_ERR_SIZE;
    int ns = 0, nr = 0;
    if (!li_ssm_scan_layout(N, vdim, &ns, &nr)) return LI_ERR_SIZE;
    const bool chunked = max_q_len > Q;
    int max_chunks = 0;
    int* chunk_tab = nullptr;
    float *carry = nullptr, *decay = nullptr;
    if (chunked) {
        const long need = li_ssm_scan_work_bytes(T, segs, heads, vdim, N, Q, &max_chunks);
        if (!work || work_bytes < need || ((uintptr_t)work % 16)) return LI_ERR_SIZE;
        chunk_tab = (int*)work;
        const long ints = ((3L * max_chunks + segs + 1 + 3) / 4) * 4;
        carry = (float*)work + ints;
        decay = carry + (size_t)max_chunks * heads * N * vdim;
    }
    const bool aligned = ((uintptr_t)state | (uintptr_t)y | (uintptr_t)carry) % 16 == 0 && y_stride % 4 == 0;
    if (chunked && fixed_a && G == heads && !Dw && aligned && Q == RET_Q && N % 4 == 0 && vdim % 4 == 0 && xbc_stride % 4 == 0 && ((uintptr_t)xbc % 16) == 0)
        return retention_launch(xbc, xbc_stride, state, slots, q_start, q_len, chunk_tab, carry, y, y_stride, heads, vdim, N, segs,
                                max_chunks, fixed_a, fixed_dt, silu_in, stream);
    int qs = 0, qr = 0;
    if (aligned && ssm_quad_layout(N, vdim, &qs, &qr)) {
        // heads that share no B and C have a block of four waves each: columns are spread over more lanes until all four work
        while (!chunked && G == heads && qs < 16 && qr > 4 && vdim <= 2 * (256 / qs)) { qs *= 2; qr /= 2; }
#define SSM_QUAD(NR_, NS_)                                                                                                \
    if (qr == NR_ && qs == NS_)                                                                                           \
        return ssm_launch<NR_, NS_, true>(silu_in, xbc, xbc_stride, dt_raw, dt_stride, dt_bias, A_log, Dw, state, slots, q_start, q_len, \
                                          chunk_tab, carry, decay, y, y_stride, heads, vdim, N, G, Q, segs, max_chunks, chunked, fixed_a, fixed_dt, stream);
        SSM_QUAD(4, 2) SSM_QUAD(8, 2) SSM_QUAD(16, 2) SSM_QUAD(32, 2)
        SSM_QUAD(4, 4) SSM_QUAD(8, 4) SSM_QUAD(16, 4) SSM_QUAD(32, 4)
        SSM_QUAD(4, 8) SSM_QUAD(8, 8) SSM_QUAD(16, 8) SSM_QUAD(32, 8)
        SSM_QUAD(4, 16) SSM_QUAD(8, 16) SSM_QUAD(16, 16) SSM_QUAD(32, 16)
#undef SSM_QUAD
    }
#define SSM_GO(NR_, NS_)                                                                                                  \
    if (nr == NR_ && ns == NS_)                                                                                           \
        return ssm_launch<NR_, NS_, false>(silu_in, xbc, xbc_stride, dt_raw, dt_stride, dt_bias, A_log, Dw, state, slots, q_start, q_len,    \
                                    chunk_tab, carry, decay, y, y_stride, heads, vdim, N, G, Q, segs, max_chunks, chunked, fixed_a, fixed_dt, stream);
    SSM_GO(16, 1) SSM_GO(32, 1) SSM_GO(64, 1) SSM_GO(128, 1)
    SSM_GO(16, 2) SSM_GO(32, 2) SSM_GO(64, 2) SSM_GO(128, 2)
    SSM_GO(16, 4) SSM_GO(32, 4) SSM_GO(64, 4)
#undef SSM_GO
    return LI_ERR_SIZE;
}

// ------------------------------------------------------------------------------------ gated delta rule
// Per head, with a state S of N x vdim values:  S <- g_t S;  u = beta_t (v_t - S^T k_t);  S <- S + k_t u^T;
// o_t = S^T q_t (the read-out sees the token's own write).  k_t and q_t are made unit vectors here
// (x / sqrt(sum x^2 + 1e-6)), q_t times q_scale; beta_t = sigmoid(b_t); g_t = exp(-exp(A_log) softplus(a_t + dt_bias)).
// Groups of heads share k and q.  A column of the state evolves by itself given the token's k, q, g, beta and its
// own v, so the layout is the state-space recurrence's: a lane owns CW neighbouring columns x NR state values,
// the NS slices of a column are neighbouring lanes that add up their shares of S^T k and of S^T q, a wave is
// 64 CW / NS columns of one head, the four waves of a block belong to ONE group and share k_t and q_t, which lie
// in LDS DR_TB tokens at a time (normed there: sixteen lanes a token add the squares in a fixed order).
// Rows of xkq: [v: heads x vdim | k: G x N | q: G x N]; rows of ba: [b: heads | a: heads].
#define DR_TB 16

// The sum over NS neighbouring lanes (NS = 1, 2, 4, 8, 16), in every lane of the group, by lane moves inside the vector
// ALU: quad_perm [1,0,3,2] and [2,3,0,1], then row_half_mirror and row_mirror (whose partners hold the other half's sum).
template <int CTRL> __device__ __forceinline__ float lane_move(float v) {
    return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xF, 0xF, true));
}
template <int NS> __device__ __forceinline__ float lanes_sum(float v) {
    if constexpr (NS >= 2) v += lane_move<0xB1>(v);
    if constexpr (NS >= 4) v += lane_move<0x4E>(v);
    if constexpr (NS >= 8) v += lane_move<0x141>(v);
    if constexpr (NS >= 16) v += lane_move<0x140>(v);
    return v;
}

//
// A step's portion of a request is cut into chunks of Q tokens that run side by side, as the state-space recurrence's
// are.  Here a token's step is S <- A_t S + beta_t k_t v_t^T with the MATRIX A_t = g_t (I - beta_t k_t k_t^T), so what a
// chunk does to the state it starts from is a matrix P = A_last ... A_first beside the state S_own that the chunk alone
// builds up from zero:
//   MODE 1: S_own of every chunk but a request's last, and P: its column j is what the recurrence, fed v = 0, makes of
//           the unit vector e_j, so P is N more columns of the same kernel (stored transposed: PT[j][n]);
//   the carry kernel: the state with which every chunk begins, chunk after chunk: S_in(c + 1) = P_c S_in(c) + S_own(c);
//   MODE 0: the recurrence itself from that state, with the outputs; the last chunk leaves the request's state.
// A portion of at most Q tokens (a decoding step) is MODE 0 alone, from the request's state.

template <int NR, int NS, int CW, int MODE>
__global__ __launch_bounds__(64 * SSM_WAVES) void delta_scan_kernel(
    const float* __restrict__ xkq, long x_stride, const float* __restrict__ ba, long ba_stride,
    const float* __restrict__ dt_bias, const float* __restrict__ A_log, float* __restrict__ state,
    const int* __restrict__ slots, const int* __restrict__ q_start, const int* __restrict__ q_len,
    const int* __restrict__ chunk_seg, const int* __restrict__ chunk_idx, float* __restrict__ carry, float* __restrict__ pmat,
    float* __restrict__ y, long y_stride, int heads, int vdim, int N, int G, int Q, float q_scale) {
    constexpr int NP = NR * NS, PW = 64 * CW / NS;
    extern __shared__ __align__(16) float lds[];
    float* sK = lds;                                   // [DR_TB][NP]
    float* sQ = sK + DR_TB * NP;                       // [DR_TB][NP]
    float* sX = sQ + DR_TB * NP;                       // [SSM_WAVES][DR_TB][PW]
    float* sBeta = sX + SSM_WAVES * DR_TB * PW;        // [SSM_WAVES][DR_TB]
    float* sG = sBeta + SSM_WAVES * DR_TB;             // [SSM_WAVES][DR_TB]
    const int bx = blockIdx.x;
    const int seg = chunk_seg ? chunk_seg[bx] : bx;
    if (seg < 0) return;
    const int c = chunk_seg ? chunk_idx[bx] : 0;
    const int L = q_len[seg], first = c * Q;
    if (first >= L) return;
    const int ntok = chunk_seg ? ((L - first < Q) ? L - first : Q) : L;
    const bool last = first + ntok >= L;
    if (MODE == 1 && last) return;                      // nobody needs the last chunk's own state
    const int t0 = q_start[seg] + first;
    // units of a head: blocks of PW value columns, and in MODE 1 behind them blocks of PW columns of P
    const int hpg = heads / G, PSV = (vdim + PW - 1) / PW, PS = PSV + (MODE == 1 ? (N + PW - 1) / PW : 0);
    const int U = hpg * PS, ublocks = (U + SSM_WAVES - 1) / SSM_WAVES;
    const int g = blockIdx.y / ublocks, ub = blockIdx.y % ublocks;
    const int w = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int unit = ub * SSM_WAVES + w;
    const bool active = unit < U;
    const int head = g * hpg + (active ? unit / PS : 0), sub = active ? unit % PS : 0;
    const bool is_p = MODE == 1 && sub >= PSV;
    const int pbase = (is_p ? sub - PSV : sub) * PW, ncols = is_p ? N : vdim;
    const int pq = lane / NS, s = lane % NS, p = pbase + CW * pq;       // the first of the lane's columns
    const int inner = heads * vdim;
    float* st = state + ((size_t)slots[seg] * heads + head) * N * vdim;
    const float* src = chunk_seg ? carry + ((size_t)bx * heads + head) * N * vdim : st;
    float S[NR][CW];
#pragma unroll
    for (int r = 0; r < NR; ++r) {
        const int n = s * NR + r;
        if (MODE == 1) {
#pragma unroll
            for (int cc = 0; cc < CW; ++cc) S[r][cc] = (is_p && n == p + cc) ? 1.f : 0.f;
        } else if constexpr (CW == 4) {
            const float4 v4 = (active && n < N && p < vdim) ? *reinterpret_cast<const float4*>(src + (size_t)n * vdim + p)
                                                            : float4{0.f, 0.f, 0.f, 0.f};
            S[r][0] = v4.x; S[r][1] = v4.y; S[r][2] = v4.z; S[r][3] = v4.w;
        } else {
#pragma unroll
            for (int cc = 0; cc < CW; ++cc) S[r][cc] = (active && n < N && p + cc < vdim) ? src[(size_t)n * vdim + p + cc] : 0.f;
        }
    }
    for (int b0 = 0; b0 < ntok; b0 += DR_TB) {
        __syncthreads();
        for (int i = threadIdx.x; i < DR_TB * NP; i += 64 * SSM_WAVES) {
            const int tt = i / NP, n = i % NP;
            const bool ok = b0 + tt < ntok && n < N;
            const float* row = xkq + (size_t)(t0 + b0 + tt) * x_stride + inner + (size_t)g * N + n;
            sK[i] = ok ? row[0] : 0.f;
            sQ[i] = ok ? row[(size_t)G * N] : 0.f;
        }
        if (active) {
            for (int i = lane; i < DR_TB * PW; i += 64) {
                const int tt = i / PW, pp = pbase + i % PW;
                const bool ok = !is_p && b0 + tt < ntok && pp < vdim;
                sX[(w * DR_TB + tt) * PW + i % PW] = ok ? xkq[(size_t)(t0 + b0 + tt) * x_stride + (size_t)head * vdim + pp] : 0.f;
            }
            if (lane < DR_TB) {
                const bool ok = b0 + lane < ntok;
                const float* r2 = ba + (size_t)(t0 + b0 + (ok ? lane : 0)) * ba_stride;
                sBeta[w * DR_TB + lane] = ok ? 1.0f / (1.0f + expf(-r2[head])) : 0.f;
                sG[w * DR_TB + lane] = ok ? expf(-expf(A_log[head]) * softplus_f32(r2[heads + head] + dt_bias[head])) : 1.f;
            }
        }
        __syncthreads();
        {   // unit vectors: token tt = thread / 16, sixteen neighbouring lanes share its N values
            const int tt = threadIdx.x >> 4, part = threadIdx.x & 15;
            float sk = 0.f, sq = 0.f;
            for (int n = part; n < NP; n += 16) {
                const float kv = sK[tt * NP + n], qv = sQ[tt * NP + n];
                sk = fmaf(kv, kv, sk);
                sq = fmaf(qv, qv, sq);
            }
#pragma unroll
            for (int o = 1; o < 16; o <<= 1) {
                sk += __shfl_xor(sk, o, LI_WAVE);
                sq += __shfl_xor(sq, o, LI_WAVE);
            }
            const float ik = 1.0f / sqrtf(sk + 1e-6f), iq = q_scale / sqrtf(sq + 1e-6f);
            for (int n = part; n < NP; n += 16) {
                sK[tt * NP + n] *= ik;
                sQ[tt * NP + n] *= iq;
            }
        }
        __syncthreads();
        if (!active) continue;
        const int nt = (ntok - b0 < DR_TB) ? ntok - b0 : DR_TB;
        for (int tt = 0; tt < nt; ++tt) {
            const float gd = sG[w * DR_TB + tt], beta = sBeta[w * DR_TB + tt];
            float xv[CW];
#pragma unroll
            for (int cc = 0; cc < CW; ++cc) xv[cc] = sX[(w * DR_TB + tt) * PW + CW * pq + cc];
            const float4* Kp = reinterpret_cast<const float4*>(sK + tt * NP + s * NR);
            const float4* Qp = reinterpret_cast<const float4*>(sQ + tt * NP + s * NR);
            float ks[CW];
#pragma unroll
            for (int cc = 0; cc < CW; ++cc) ks[cc] = 0.f;
#pragma unroll
            for (int r4 = 0; r4 < NR / 4; ++r4) {
                const float4 kv = Kp[r4];
                const float kk[4] = {kv.x, kv.y, kv.z, kv.w};
#pragma unroll
                for (int j = 0; j < 4; ++j)
#pragma unroll
                    for (int cc = 0; cc < CW; ++cc) ks[cc] = fmaf(S[4 * r4 + j][cc], kk[j], ks[cc]);
            }
#pragma unroll
            for (int cc = 0; cc < CW; ++cc) ks[cc] = lanes_sum<NS>(ks[cc]);
            float u[CW], ov[CW];
#pragma unroll
            for (int cc = 0; cc < CW; ++cc) { u[cc] = beta * (xv[cc] - gd * ks[cc]); ov[cc] = 0.f; }
#pragma unroll
            for (int r4 = 0; r4 < NR / 4; ++r4) {
                const float4 kv = Kp[r4];
                const float kk[4] = {kv.x, kv.y, kv.z, kv.w};
                float qs[4] = {0.f, 0.f, 0.f, 0.f};
                if (MODE == 0) { const float4 qv = Qp[r4]; qs[0] = qv.x; qs[1] = qv.y; qs[2] = qv.z; qs[3] = qv.w; }
#pragma unroll
                for (int j = 0; j < 4; ++j)
#pragma unroll
                    for (int cc = 0; cc < CW; ++cc) {
                        const float nv = fmaf(gd, S[4 * r4 + j][cc], kk[j] * u[cc]);
                        S[4 * r4 + j][cc] = nv;
                        if (MODE == 0) ov[cc] = fmaf(nv, qs[j], ov[cc]);
                    }
            }
            if (MODE == 0) {
#pragma unroll
                for (int cc = 0; cc < CW; ++cc) ov[cc] = lanes_sum<NS>(ov[cc]);
                if (s == 0) {
                    float* yr = y + (size_t)(t0 + b0 + tt) * y_stride + (size_t)head * vdim + p;
                    if constexpr (CW == 4) {
                        if (p < vdim) *reinterpret_cast<float4*>(yr) = float4{ov[0], ov[1], ov[2], ov[3]};
                    } else {
#pragma unroll
                        for (int cc = 0; cc < CW; ++cc) if (p + cc < vdim) yr[cc] = ov[cc];
                    }
                }
            }
        }
    }
    if (!active) return;
    if (MODE == 1 && is_p) {                            // PT[j][n]: the lane's columns j, its n values side by side
        float* pt = pmat + ((size_t)bx * heads + head) * N * N;
#pragma unroll
        for (int cc = 0; cc < CW; ++cc)
#pragma unroll
            for (int r = 0; r < NR; ++r) {
                const int n = s * NR + r;
                if (n < N && p + cc < N) pt[(size_t)(p + cc) * N + n] = S[r][cc];
            }
        return;
    }
    float* dst = MODE == 1 ? carry + ((size_t)bx * heads + head) * N * vdim : (last ? st : nullptr);
    if (!dst) return;
#pragma unroll
    for (int r = 0; r < NR; ++r) {
        const int n = s * NR + r;
        if (n >= N) continue;
        if constexpr (CW == 4) {
            if (p < vdim) *reinterpret_cast<float4*>(dst + (size_t)n * vdim + p) = float4{S[r][0], S[r][1], S[r][2], S[r][3]};
        } else {
#pragma unroll
            for (int cc = 0; cc < CW; ++cc) if (p + cc < vdim) dst[(size_t)n * vdim + p + cc] = S[r][cc];
        }
    }
    (void)ncols;
}

// carry[chunk] holds what the chunk alone built up from zero, pmat[chunk] its matrix (transposed); afterwards carry[chunk]
// holds the state with which the chunk begins.  A block takes a request, a head and 16 columns of the state, which lie in
// LDS, chunk after chunk: S_in(c + 1) = P_c S_in(c) + S_own(c), on the float32 matrix cores (v_mfma_f32_16x16x4_f32: row
// operand P, one value a lane (row lane % 16, k lane / 16), which lie side by side in a row of the stored transpose; column
// operand the state from LDS; the accumulator starts as S_own and holds rows 4 (lane / 16) + r of column lane % 16).  A
// wave owns RT tiles of 16 rows; P comes in groups of 64 k's, and a group is on its way while the one before it is used,
// across the chunks' borders too (P and S_own do not depend on the state).  Rows and k's past N: loads are clamped, the
// state's rows past N are zeros in LDS, and results past N are never stored.
#define DC_GROUP 16                 // matrix instructions (4 k's each) of a group
typedef float dc_f32x4 __attribute__((ext_vector_type(4)));
template <int RT>
__global__ __launch_bounds__(256) void delta_carry_kernel(
    float* __restrict__ carry, const float* __restrict__ pmat, const float* __restrict__ state, const int* __restrict__ slots,
    const int* __restrict__ q_len, const int* __restrict__ chunk_first, int heads, int vdim, int N, int Q) {
    extern __shared__ float run[];                      // [N rounded up to 64][16]
    const int seg = blockIdx.x, head = blockIdx.y, lane = threadIdx.x & 63, w = threadIdx.x >> 6;
    const int cl = lane & 15, kq = lane >> 4, col = blockIdx.z * 16 + cl;
    const int nch = (q_len[seg] + Q - 1) / Q, base = chunk_first[seg];
    const bool on = col < vdim;
    const int groups = (N + 4 * DC_GROUP - 1) / (4 * DC_GROUP);
    const float* stp = state + ((size_t)slots[seg] * heads + head) * N * vdim;
    for (int i = threadIdx.x; i < groups * 4 * DC_GROUP * 16; i += 256) {
        const int n = i / 16, cc = blockIdx.z * 16 + i % 16;
        run[i] = (n < N && cc < vdim) ? stp[(size_t)n * vdim + cc] : 0.f;
    }
    int arow[RT], crow[RT];                             // this lane's row of P (operand) and its first row of the result
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
        const int r = 16 * (w * RT + rt);
        arow[rt] = r + cl < N ? r + cl : N - 1;
        crow[rt] = r + 4 * kq;
    }
    float pa[RT][DC_GROUP], pb[RT][DC_GROUP], own[RT][4];
    dc_f32x4 acc[RT];
    const int steps = (nch - 1) * groups;               // a request's last chunk only takes the state it begins with
    auto fetch = [&](int st, float (&p)[RT][DC_GROUP]) {
        if (st >= steps) return;
        const float* pt = pmat + ((size_t)(base + st / groups) * heads + head) * N * N;
        const int k0 = (st % groups) * 4 * DC_GROUP + kq;
#pragma unroll
        for (int x = 0; x < DC_GROUP; ++x) {
            const int k = k0 + 4 * x < N ? k0 + 4 * x : N - 1;
#pragma unroll
            for (int rt = 0; rt < RT; ++rt) p[rt][x] = pt[(size_t)k * N + arow[rt]];
        }
    };
    auto own_of = [&](int k) {
        if (k + 1 >= nch) return;
        const float* at = carry + ((size_t)(base + k) * heads + head) * N * vdim + (on ? col : 0);
#pragma unroll
        for (int rt = 0; rt < RT; ++rt)
#pragma unroll
            for (int r = 0; r < 4; ++r) own[rt][r] = at[(size_t)(crow[rt] + r < N ? crow[rt] + r : N - 1) * vdim];
    };
    auto leave = [&](int k) {                           // the state with which chunk k begins
        float* at = carry + ((size_t)(base + k) * heads + head) * N * vdim + col;
#pragma unroll
        for (int rt = 0; rt < RT; ++rt)
#pragma unroll
            for (int r = 0; r < 4; ++r)
                if (on && crow[rt] + r < N) at[(size_t)(crow[rt] + r) * vdim] = run[(crow[rt] + r) * 16 + cl];
    };
    auto step = [&](int st, const float (&p)[RT][DC_GROUP]) {
        const int k = st / groups, g = st % groups;
        if (g == 0) {
#pragma unroll
            for (int rt = 0; rt < RT; ++rt)
#pragma unroll
                for (int r = 0; r < 4; ++r) acc[rt][r] = own[rt][r];
            own_of(k + 1);
            leave(k);
        }
#pragma unroll
        for (int x = 0; x < DC_GROUP; ++x) {
            const float b = run[(g * 4 * DC_GROUP + 4 * x + kq) * 16 + cl];
#pragma unroll
            for (int rt = 0; rt < RT; ++rt) acc[rt] = __builtin_amdgcn_mfma_f32_16x16x4f32(p[rt][x], b, acc[rt], 0, 0, 0);
        }
        if (g == groups - 1) {
            __syncthreads();
#pragma unroll
            for (int rt = 0; rt < RT; ++rt)
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    if (crow[rt] + r < N) run[(crow[rt] + r) * 16 + cl] = acc[rt][r];
            __syncthreads();
        }
    };
    fetch(0, pa);
    own_of(0);
    __syncthreads();
    for (int st = 0; st < steps; st += 2) {
        fetch(st + 1, pb);
        step(st, pa);
        fetch(st + 2, pa);
        if (st + 1 < steps) step(st + 1, pb);
    }
    leave(nch - 1);
}

static void delta_carry_launch(float* carry, const float* pmat, const float* state, const int* slots, const int* q_len,
                               const int* chunk_first, int heads, int vdim, int N, int Q, int segs, hipStream_t stream) {
    const dim3 grid(segs, heads, (vdim + 15) / 16);
    const size_t lds = (size_t)((N + 4 * DC_GROUP - 1) / (4 * DC_GROUP) * 4 * DC_GROUP) * 16 * sizeof(float);
#define DC_GO(R_) delta_carry_kernel<R_><<<grid, 256, lds, stream>>>(carry, pmat, state, slots, q_len, chunk_first, heads, vdim, N, Q)
    if (N <= 64) DC_GO(1); else if (N <= 128) DC_GO(2); else DC_GO(4);
#undef DC_GO
}

template <int NR, int NS, int CW>
static int delta_launch(const float* xkq, long x_stride, const float* ba, long ba_stride, const float* dt_bias, const float* A_log,
                        float* state, const int* slots, const int* q_start, const int* q_len, int* chunk_tab, float* carry,
                        float* pmat, float* y, long y_stride, int heads, int vdim, int N, int G, int Q, float q_scale, int segs,
                        int max_chunks, bool chunked, hipStream_t stream) {
    constexpr int NP = NR * NS, PW = 64 * CW / NS;
    const size_t lds = (size_t)(2 * DR_TB * NP + SSM_WAVES * DR_TB * PW + 2 * SSM_WAVES * DR_TB) * sizeof(float);
    const int hpg = heads / G, PSV = (vdim + PW - 1) / PW, PSP = (N + PW - 1) / PW;
    const int ub0 = (hpg * PSV + SSM_WAVES - 1) / SSM_WAVES, ub1 = (hpg * (PSV + PSP) + SSM_WAVES - 1) / SSM_WAVES;
    if (!chunked) {
        delta_scan_kernel<NR, NS, CW, 0><<<dim3(segs, G * ub0), 64 * SSM_WAVES, lds, stream>>>(
            xkq, x_stride, ba, ba_stride, dt_bias, A_log, state, slots, q_start, q_len, nullptr, nullptr, nullptr, nullptr,
            y, y_stride, heads, vdim, N, G, Q, q_scale);
        return li_launch_status();
    }
    int* chunk_seg = chunk_tab;
    int* chunk_idx = chunk_tab + max_chunks;
    int* chunk_first = chunk_tab + 2 * max_chunks;
    ssm_chunk_index_kernel<<<1, 256, 0, stream>>>(q_len, segs, Q, max_chunks, chunk_seg, chunk_idx, chunk_first);
    delta_scan_kernel<NR, NS, CW, 1><<<dim3(max_chunks, G * ub1), 64 * SSM_WAVES, lds, stream>>>(
        xkq, x_stride, ba, ba_stride, dt_bias, A_log, state, slots, q_start, q_len, chunk_seg, chunk_idx, carry, pmat,
        y, y_stride, heads, vdim, N, G, Q, q_scale);
    delta_carry_launch(carry, pmat, state, slots, q_len, chunk_first, heads, vdim, N, Q, segs, stream);
    delta_scan_kernel<NR, NS, CW, 0><<<dim3(max_chunks, G * ub0), 64 * SSM_WAVES, lds, stream>>>(
        xkq, x_stride, ba, ba_stride, dt_bias, A_log, state, slots, q_start, q_len, chunk_seg, chunk_idx, carry, pmat,
        y, y_stride, heads, vdim, N, G, Q, q_scale);
    return li_launch_status();
}

// 1 if the recurrence has a layout for a state of N values a column (the state-space recurrence's layouts)
extern "C" int li_delta_scan_takes(int N, int vdim) { return li_ssm_scan_layout(N, vdim, nullptr, nullptr); }

// Chunks that a step of T tokens in `segs` portions can have at most, and the bytes of the tables, states and matrices
// that the chunked form keeps in the workspace.
extern "C" long li_delta_scan_work_bytes(int T, int segs, int heads, int vdim, int N, int Q, int* max_chunks) {
    const long mc = (long)T / Q + segs;
    if (max_chunks) *max_chunks = (int)mc;
    const long ints = ((3 * mc + segs + 1 + 3) / 4) * 4;
    return ints * 4 + mc * heads * ((long)N * vdim + (long)N * N) * 4;
}

extern "C" int li_delta_scan(const float* xkq, long x_stride, const float* ba, long ba_stride, const float* dt_bias,
                             const float* A_log, float* state, const int* slots, const int* q_start, const int* q_len,
                             float* y, long y_stride, int heads, int vdim, int N, int G, float q_scale, int Q, int T, int segs,
                             int max_q_len, void* work, long work_bytes, hipStream_t stream) {
    if (T <= 0 || segs <= 0 || heads <= 0 || G <= 0 || heads % G || vdim <= 0 || N <= 0 || N > 256 || Q <= 0 || max_q_len <= 0 ||
        x_stride < (long)heads * vdim + 2L * G * N || ba_stride < 2L * heads || y_stride < (long)heads * vdim)
        return LI_ERR_SIZE;
    const bool chunked = max_q_len > Q;
    int max_chunks = 0;
    int* chunk_tab = nullptr;
    float *carry = nullptr, *pmat = nullptr;
    if (chunked) {
        const long need = li_delta_scan_work_bytes(T, segs, heads, vdim, N, Q, &max_chunks);
        if (!work || work_bytes < need || ((uintptr_t)work % 16)) return LI_ERR_SIZE;
        chunk_tab = (int*)work;
        const long ints = ((3L * max_chunks + segs + 1 + 3) / 4) * 4;
        carry = (float*)work + ints;
        pmat = carry + (size_t)max_chunks * heads * N * vdim;
    }
#define DR_ARGS xkq, x_stride, ba, ba_stride, dt_bias, A_log, state, slots, q_start, q_len, chunk_tab, carry, pmat, y, y_stride, heads, \
                vdim, N, G, Q, q_scale, segs, max_chunks, chunked, stream
    const bool aligned = ((uintptr_t)state | (uintptr_t)y | (uintptr_t)carry) % 16 == 0 && y_stride % 4 == 0;
    int qs = 0, qr = 0;
    if (aligned && ssm_quad_layout(N, vdim, &qs, &qr)) {
#define DR_QUAD(NR_, NS_) if (qr == NR_ && qs == NS_) return delta_launch<NR_, NS_, 4>(DR_ARGS);
        DR_QUAD(4, 2) DR_QUAD(8, 2) DR_QUAD(16, 2) DR_QUAD(32, 2)
        DR_QUAD(4, 4) DR_QUAD(8, 4) DR_QUAD(16, 4) DR_QUAD(32, 4)
        DR_QUAD(4, 8) DR_QUAD(8, 8) DR_QUAD(16, 8) DR_QUAD(32, 8)
        DR_QUAD(4, 16) DR_QUAD(8, 16) DR_QUAD(16, 16)
#undef DR_QUAD
    }
    int ns = 0, nr = 0;
    if (!li_ssm_scan_layout(N, vdim, &ns, &nr)) return LI_ERR_SIZE;
#define DR_GO(NR_, NS_) if (nr == NR_ && ns == NS_) return delta_launch<NR_, NS_, 1>(DR_ARGS);
    DR_GO(16, 1) DR_GO(32, 1) DR_GO(64, 1) DR_GO(128, 1)
    DR_GO(16, 2) DR_GO(32, 2) DR_GO(64, 2) DR_GO(128, 2)
    DR_GO(16, 4) DR_GO(32, 4) DR_GO(64, 4)
#undef DR_GO
#undef DR_ARGS
    return LI_ERR_SIZE;
}

// ------------------------------------------------------------------------------------ delta rule, channel by channel
// Per head, with a state S of N x vdim values and the unit key u_t = k_t / sqrt(sum k_t^2 + 1e-6):
//   S <- diag(w_t) S - (a_t * u_t) (u_t^T S) + k_t v_t^T      (both terms read the old S),      o_t = S^T r_t,
// with w_t = exp(-exp(-1/2) sigmoid(low_t)) and a_t = sigmoid(araw_t), one number a head and key channel each.  With
// k = |k| u the step of a state value is  S[n] <- w[n] S[n] + u[n] (|k| v - a[n] (u^T S)):  u, a, w and r are all a token
// needs beside its |k| v.  A token's step is again S <- A_t S + k_t v_t^T with a matrix A_t = diag(w_t) - (a_t * u_t) u_t^T,
// so a portion runs as chunks side by side exactly as the gated delta rule's does (same modes, same carry kernel), and
// the layout is the same: a lane owns CW neighbouring columns x NR state values, NS neighbouring lanes share a column.
// No heads share keys here: the waves of a block are columns of ONE head (as many waves as the head has units, up to
// four) and share u, a, w and r, which are worked out when a block of CD_TB tokens is staged in LDS; the next block's raw
// values are on their way in registers meanwhile.
// Rows of x: [r: heads x N | k: heads x N | v: heads x vdim | a: heads x N]; rows of low: heads x N.
#define CD_DECAY 0.6065306597126334f               // exp(-1/2)
#define CD_TB 8                                    // tokens staged at a time

template <int NR, int NS, int CW, int NW, int MODE>
__global__ __launch_bounds__(64 * NW) void channel_delta_kernel(
    const float* __restrict__ x, long x_stride, const float* __restrict__ low, long low_stride, float* __restrict__ state,
    const int* __restrict__ slots, const int* __restrict__ q_start, const int* __restrict__ q_len,
    const int* __restrict__ chunk_seg, const int* __restrict__ chunk_idx, float* __restrict__ carry, float* __restrict__ pmat,
    float* __restrict__ y, long y_stride, int heads, int vdim, int N, int Q) {
    constexpr int NP = NR * NS, PW = 64 * CW / NS, TB = CD_TB, NT = 64 * NW;
    constexpr int IT = (TB * NP + NT - 1) / NT, IV = (TB * PW + 63) / 64;      // staged values a thread (keys' vectors; a wave's v)
    __shared__ __attribute__((aligned(16))) float sU[TB * NP];
    __shared__ __attribute__((aligned(16))) float sA[TB * NP];
    __shared__ __attribute__((aligned(16))) float sW[TB * NP];
    __shared__ __attribute__((aligned(16))) float sR[MODE == 0 ? TB * NP : 4];
    __shared__ __attribute__((aligned(16))) float sX[NW * TB * PW];
    __shared__ float sN[TB];                            // |k|
    const int bx = blockIdx.x;
    const int seg = chunk_seg ? chunk_seg[bx] : bx;
    if (seg < 0) return;
    const int c = chunk_seg ? chunk_idx[bx] : 0;
    const int L = q_len[seg], first = c * Q;
    if (first >= L) return;
    const int ntok = chunk_seg ? ((L - first < Q) ? L - first : Q) : L;
    const bool last = first + ntok >= L;
    if (MODE == 1 && last) return;                      // nobody needs the last chunk's own state
    const int t0 = q_start[seg] + first;
    // units of a head: blocks of PW value columns, and in MODE 1 behind them blocks of PW columns of P
    const int PSV = (vdim + PW - 1) / PW, PS = PSV + (MODE == 1 ? (N + PW - 1) / PW : 0);
    const int ublocks = (PS + NW - 1) / NW;
    const int head = blockIdx.y / ublocks, ub = blockIdx.y % ublocks;
    const int w = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int unit = ub * NW + w;
    const bool active = unit < PS;
    const int sub = active ? unit : 0;
    const bool is_p = MODE == 1 && sub >= PSV;
    const int pbase = (is_p ? sub - PSV : sub) * PW;
    const int pq = lane / NS, s = lane % NS, p = pbase + CW * pq;       // the first of the lane's columns
    const long n_key = (long)heads * N;
    const float* xr0 = x + (size_t)head * N;
    const float* xv0 = x + 2 * n_key + (size_t)head * vdim;
    const float* xa0 = x + 2 * n_key + (long)heads * vdim + (size_t)head * N;
    const float* lw0 = low + (size_t)head * N;
    float* st = state + ((size_t)slots[seg] * heads + head) * N * vdim;
    const float* src = chunk_seg ? carry + ((size_t)bx * heads + head) * N * vdim : st;
    // a block of tokens on its way: raw values in registers (a place past the end reads a valid one and is blanked below)
    float gk[IT], ga[IT], gl[IT], gr[IT], gv[IV];
    auto fetch = [&](int b0) {
#pragma unroll
        for (int it = 0; it < IT; ++it) {
            const int i = threadIdx.x + NT * it, tt = i / NP, n = i % NP;
            const size_t row = (size_t)(t0 + (tt < TB && b0 + tt < ntok ? b0 + tt : 0));
            const int nn = n < N ? n : 0;
            gk[it] = xr0[row * x_stride + n_key + nn];
            ga[it] = xa0[row * x_stride + nn];
            gl[it] = lw0[row * low_stride + nn];
            if (MODE == 0) gr[it] = xr0[row * x_stride + nn];
        }
#pragma unroll
        for (int it = 0; it < IV; ++it) {
            const int i = lane + 64 * it, tt = i / PW, pp = pbase + i % PW;
            const size_t row = (size_t)(t0 + (tt < TB && b0 + tt < ntok ? b0 + tt : 0));
            gv[it] = xv0[row * x_stride + (!is_p && pp < vdim ? pp : 0)];
        }
    };
    fetch(0);
    float S[NR][CW];
#pragma unroll
    for (int r = 0; r < NR; ++r) {
        const int n = s * NR + r;
        if (MODE == 1) {
#pragma unroll
            for (int cc = 0; cc < CW; ++cc) S[r][cc] = (is_p && n == p + cc) ? 1.f : 0.f;
        } else if constexpr (CW == 4) {
            const float4 v4 = (active && n < N && p < vdim) ? *reinterpret_cast<const float4*>(src + (size_t)n * vdim + p)
                                                            : float4{0.f, 0.f, 0.f, 0.f};
            S[r][0] = v4.x; S[r][1] = v4.y; S[r][2] = v4.z; S[r][3] = v4.w;
        } else {
#pragma unroll
            for (int cc = 0; cc < CW; ++cc) S[r][cc] = (active && n < N && p + cc < vdim) ? src[(size_t)n * vdim + p + cc] : 0.f;
        }
    }
    for (int b0 = 0; b0 < ntok; b0 += TB) {
        __syncthreads();
#pragma unroll
        for (int it = 0; it < IT; ++it) {
            const int i = threadIdx.x + NT * it, tt = i / NP, n = i % NP;
            const bool ok = b0 + tt < ntok && n < N;
            if (TB * NP % NT == 0 || i < TB * NP) {
                sU[i] = ok ? gk[it] : 0.f;
                sA[i] = ok ? 1.0f / (1.0f + expf(-ga[it])) : 0.f;
                sW[i] = ok ? expf(-CD_DECAY / (1.0f + expf(-gl[it]))) : 1.f;
                if (MODE == 0) sR[i] = ok ? gr[it] : 0.f;
            }
        }
#pragma unroll
        for (int it = 0; it < IV; ++it) {
            const int i = lane + 64 * it, tt = i / PW, pp = pbase + i % PW;
            if (TB * PW % 64 == 0 || i < TB * PW) sX[w * TB * PW + i] = (!is_p && b0 + tt < ntok && pp < vdim) ? gv[it] : 0.f;
        }
        __syncthreads();
        // unit keys: sixteen neighbouring lanes share a token's N values
        for (int tt = threadIdx.x >> 4; tt < TB; tt += NT / 16) {
            const int part = threadIdx.x & 15;
            float sk = 0.f;
            for (int n = part; n < NP; n += 16) sk = fmaf(sU[tt * NP + n], sU[tt * NP + n], sk);
            sk = lanes_sum<16>(sk);
            const float len = sqrtf(sk + 1e-6f), inv = 1.0f / len;
            for (int n = part; n < NP; n += 16) sU[tt * NP + n] *= inv;
            if (part == 0) sN[tt] = len;
        }
        __syncthreads();
        if (b0 + TB < ntok) fetch(b0 + TB);              // (on its way while this block is worked on)
        if (!active) continue;
        const int nt = (ntok - b0 < TB) ? ntok - b0 : TB;
        for (int tt = 0; tt < nt; ++tt) {
            const float len = sN[tt];
            float vn[CW], ks[CW], ov[CW];
#pragma unroll
            for (int cc = 0; cc < CW; ++cc) { vn[cc] = len * sX[(w * TB + tt) * PW + CW * pq + cc]; ks[cc] = 0.f; ov[cc] = 0.f; }
            const float4* Up = reinterpret_cast<const float4*>(sU + tt * NP + s * NR);
            const float4* Ap = reinterpret_cast<const float4*>(sA + tt * NP + s * NR);
            const float4* Wp = reinterpret_cast<const float4*>(sW + tt * NP + s * NR);
            const float4* Rp = reinterpret_cast<const float4*>(sR + (MODE == 0 ? tt * NP + s * NR : 0));
#pragma unroll
            for (int r4 = 0; r4 < NR / 4; ++r4) {
                const float4 uv = Up[r4];
                const float uu[4] = {uv.x, uv.y, uv.z, uv.w};
#pragma unroll
                for (int j = 0; j < 4; ++j)
#pragma unroll
                    for (int cc = 0; cc < CW; ++cc) ks[cc] = fmaf(S[4 * r4 + j][cc], uu[j], ks[cc]);
            }
#pragma unroll
            for (int cc = 0; cc < CW; ++cc) ks[cc] = lanes_sum<NS>(ks[cc]);
#pragma unroll
            for (int r4 = 0; r4 < NR / 4; ++r4) {
                const float4 uv = Up[r4], av = Ap[r4], wv = Wp[r4];
                const float uu[4] = {uv.x, uv.y, uv.z, uv.w}, aa[4] = {av.x, av.y, av.z, av.w}, ww[4] = {wv.x, wv.y, wv.z, wv.w};
                float rr[4] = {0.f, 0.f, 0.f, 0.f};
                if (MODE == 0) { const float4 rv = Rp[r4]; rr[0] = rv.x; rr[1] = rv.y; rr[2] = rv.z; rr[3] = rv.w; }
#pragma unroll
                for (int j = 0; j < 4; ++j)
#pragma unroll
                    for (int cc = 0; cc < CW; ++cc) {
                        const float nv = fmaf(ww[j], S[4 * r4 + j][cc], uu[j] * fmaf(-aa[j], ks[cc], vn[cc]));
                        S[4 * r4 + j][cc] = nv;
                        if (MODE == 0) ov[cc] = fmaf(nv, rr[j], ov[cc]);
                    }
            }
            if (MODE == 0) {
#pragma unroll
                for (int cc = 0; cc < CW; ++cc) ov[cc] = lanes_sum<NS>(ov[cc]);
                if (s == 0) {
                    float* yr = y + (size_t)(t0 + b0 + tt) * y_stride + (size_t)head * vdim + p;
                    if constexpr (CW == 4) {
                        if (p < vdim) *reinterpret_cast<float4*>(yr) = float4{ov[0], ov[1], ov[2], ov[3]};
                    } else {
#pragma unroll
                        for (int cc = 0; cc < CW; ++cc) if (p + cc < vdim) yr[cc] = ov[cc];
                    }
                }
            }
        }
    }
    if (!active) return;
    if (MODE == 1 && is_p) {                            // PT[j][n]: the lane's columns j, its n values side by side
        float* pt = pmat + ((size_t)bx * heads + head) * N * N;
#pragma unroll
        for (int cc = 0; cc < CW; ++cc)
#pragma unroll
            for (int r = 0; r < NR; ++r) {
                const int n = s * NR + r;
                if (n < N && p + cc < N) pt[(size_t)(p + cc) * N + n] = S[r][cc];
            }
        return;
    }
    float* dst = MODE == 1 ? carry + ((size_t)bx * heads + head) * N * vdim : (last ? st : nullptr);
    if (!dst) return;
#pragma unroll
    for (int r = 0; r < NR; ++r) {
        const int n = s * NR + r;
        if (n >= N) continue;
        if constexpr (CW == 4) {
            if (p < vdim) *reinterpret_cast<float4*>(dst + (size_t)n * vdim + p) = float4{S[r][0], S[r][1], S[r][2], S[r][3]};
        } else {
#pragma unroll
            for (int cc = 0; cc < CW; ++cc) if (p + cc < vdim) dst[(size_t)n * vdim + p + cc] = S[r][cc];
        }
    }
}

// W0, W1: waves a block without and with P's columns (as many as a head of as many columns as rows has units, up to four)
template <int NR, int NS, int CW, int W0, int W1>
static int channel_delta_launch(const float* x, long x_stride, const float* low, long low_stride, float* state, const int* slots,
                                const int* q_start, const int* q_len, int* chunk_tab, float* carry, float* pmat, float* y,
                                long y_stride, int heads, int vdim, int N, int Q, int segs, int max_chunks, bool chunked,
                                hipStream_t stream) {
    constexpr int PW = 64 * CW / NS;
    const int PSV = (vdim + PW - 1) / PW, PSP = (N + PW - 1) / PW;
    const int ub0 = (PSV + W0 - 1) / W0, ub1 = (PSV + PSP + W1 - 1) / W1;
    if (!chunked) {
        channel_delta_kernel<NR, NS, CW, W0, 0><<<dim3(segs, heads * ub0), 64 * W0, 0, stream>>>(
            x, x_stride, low, low_stride, state, slots, q_start, q_len, nullptr, nullptr, nullptr, nullptr, y, y_stride, heads, vdim, N, Q);
        return li_launch_status();
    }
    int* chunk_seg = chunk_tab;
    int* chunk_idx = chunk_tab + max_chunks;
    int* chunk_first = chunk_tab + 2 * max_chunks;
    ssm_chunk_index_kernel<<<1, 256, 0, stream>>>(q_len, segs, Q, max_chunks, chunk_seg, chunk_idx, chunk_first);
    channel_delta_kernel<NR, NS, CW, W1, 1><<<dim3(max_chunks, heads * ub1), 64 * W1, 0, stream>>>(
        x, x_stride, low, low_stride, state, slots, q_start, q_len, chunk_seg, chunk_idx, carry, pmat, y, y_stride, heads, vdim, N, Q);
    delta_carry_launch(carry, pmat, state, slots, q_len, chunk_first, heads, vdim, N, Q, segs, stream);
    channel_delta_kernel<NR, NS, CW, W0, 0><<<dim3(max_chunks, heads * ub0), 64 * W0, 0, stream>>>(
        x, x_stride, low, low_stride, state, slots, q_start, q_len, chunk_seg, chunk_idx, carry, pmat, y, y_stride, heads, vdim, N, Q);
    return li_launch_status();
}

extern "C" int li_channel_delta(const float* x, long x_stride, const float* low, long low_stride, float* state, const int* slots,
                                const int* q_start, const int* q_len, float* y, long y_stride, int heads, int vdim, int N, int Q,
                                int T, int segs, int max_q_len, void* work, long work_bytes, hipStream_t stream) {
    if (T <= 0 || segs <= 0 || heads <= 0 || vdim <= 0 || N <= 0 || N > 256 || Q <= 0 || max_q_len <= 0 ||
        x_stride < 3L * heads * N + (long)heads * vdim || low_stride < (long)heads * N || y_stride < (long)heads * vdim)
        return LI_ERR_SIZE;
    const bool chunked = max_q_len > Q;
    int max_chunks = 0;
    int* chunk_tab = nullptr;
    float *carry = nullptr, *pmat = nullptr;
    if (chunked) {
        const long need = li_delta_scan_work_bytes(T, segs, heads, vdim, N, Q, &max_chunks);
        if (!work || work_bytes < need || ((uintptr_t)work % 16)) return LI_ERR_SIZE;
        chunk_tab = (int*)work;
        const long ints = ((3L * max_chunks + segs + 1 + 3) / 4) * 4;
        carry = (float*)work + ints;
        pmat = carry + (size_t)max_chunks * heads * N * vdim;
    }
#define CD_ARGS x, x_stride, low, low_stride, state, slots, q_start, q_len, chunk_tab, carry, pmat, y, y_stride, heads, vdim, N, Q,                 segs, max_chunks, chunked, stream
    // four columns a lane and rows of the state in 16-byte pieces, or (sizes that are no multiple of four) one column a lane
    const bool quad = vdim % 4 == 0 && ((uintptr_t)state | (uintptr_t)y | (uintptr_t)carry) % 16 == 0 && y_stride % 4 == 0;
#define CD_GO(NR_, NS_, W0_, W1_)                                                   \
    {                                                                               \
        if (quad) return channel_delta_launch<NR_, NS_, 4, W0_, W1_>(CD_ARGS);      \
        return channel_delta_launch<NR_, NS_, 1, 4, 4>(CD_ARGS);                    \
    }
    if (N <= 32) CD_GO(4, 8, 1, 2)
    if (N <= 64) CD_GO(8, 8, 2, 4)
    if (N <= 128) CD_GO(16, 8, 4, 4)
    CD_GO(16, 16, 4, 4)
#undef CD_GO
#undef CD_ARGS
}

// ------------------------------------------------------------------------------------ gated norm in groups
// Every group of `gs` neighbouring columns has its own root mean square.  gate_after 0: out[t, c] = w[c] * v /
// sqrt(mean of v^2 over c's group + eps) with v = y[t, c] * silu(z[t, c]): the gate comes before the norm.
// gate_after 1: out[t, c] = w[c] * y / sqrt(mean of y^2 + eps) * silu(z[t, c]): the norm sees y alone.  gate_after 2: the
// same with sigmoid(z) for silu(z).  w null: ones.
// A block a (token, group).
template <typename TO, int PER>
__global__ __launch_bounds__(256) void gated_group_norm_kernel(const float* __restrict__ y, long y_stride,
                                                               const float* __restrict__ z, long z_stride,
                                                               const float* __restrict__ w, float eps, TO* __restrict__ out,
                                                               long out_stride, int gs, int gate_after) {
    __shared__ float red[256 / LI_WAVE];
    const int t = blockIdx.x, c0 = blockIdx.y * gs;
    const float* yr = y + (size_t)t * y_stride + c0;
    const float* zr = z + (size_t)t * z_stride + c0;
    float v[PER], gt[PER];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < PER; ++i) {
        const int j = threadIdx.x + i * 256;
        float g = 0.f, sg = 0.f;
        if (j < gs) { const float zz = zr[j]; sg = (gate_after == 2 ? 1.0f : zz) / (1.0f + expf(-zz)); g = gate_after ? yr[j] : yr[j] * sg; }
        v[i] = g;
        gt[i] = gate_after ? sg : 1.f;
        ss += g * g;
    }
    for (int j = threadIdx.x + PER * 256; j < gs; j += 256) {
        const float zz = zr[j], sg = (gate_after == 2 ? 1.0f : zz) / (1.0f + expf(-zz)), g = gate_after ? yr[j] : yr[j] * sg;
        ss += g * g;
    }
    ss = block_sum<256>(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)gs + eps);
    TO* o = out + (size_t)t * out_stride + c0;
#pragma unroll
    for (int i = 0; i < PER; ++i) {
        const int j = threadIdx.x + i * 256;
        if (j < gs) store_from_float(o + j, (w ? w[c0 + j] : 1.f) * v[i] * inv * gt[i]);
    }
    for (int j = threadIdx.x + PER * 256; j < gs; j += 256) {
        const float zz = zr[j], sg = (gate_after == 2 ? 1.0f : zz) / (1.0f + expf(-zz)), g = gate_after ? yr[j] : yr[j] * sg;
        store_from_float(o + j, (w ? w[c0 + j] : 1.f) * g * inv * (gate_after ? sg : 1.f));
    }
}

// The same for narrow groups (up to 256 columns): a wave a (token, group), four of them a block.
template <typename TO>
__global__ __launch_bounds__(256) void gated_group_norm_wave_kernel(const float* __restrict__ y, long y_stride,
                                                                    const float* __restrict__ z, long z_stride,
                                                                    const float* __restrict__ w, float eps, TO* __restrict__ out,
                                                                    long out_stride, long units, int groups, int gs, int gate_after) {
    const long unit = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
    const int lane = threadIdx.x & 63;
    if (unit >= units) return;
    const long t = unit / groups;
    const int c0 = (int)(unit % groups) * gs;
    const float* yr = y + t * y_stride + c0;
    const float* zr = z + t * z_stride + c0;
    float v[4], gt[4];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int j = lane + 64 * i;
        v[i] = 0.f; gt[i] = 1.f;
        if (j < gs) {
            const float zz = zr[j], sg = (gate_after == 2 ? 1.0f : zz) / (1.0f + expf(-zz));
            v[i] = gate_after ? yr[j] : yr[j] * sg;
            if (gate_after) gt[i] = sg;
        }
        ss = fmaf(v[i], v[i], ss);
    }
    const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)gs + eps);
    TO* o = out + t * out_stride + c0;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int j = lane + 64 * i;
        if (j < gs) store_from_float(o + j, (w ? w[c0 + j] : 1.f) * v[i] * inv * gt[i]);
    }
}

extern "C" int li_gated_group_norm(const float* y, long y_stride, const float* z, long z_stride, const float* w, float eps,
                                   void* out, int out_dtype, long out_stride, int T, int n, int groups, int gate_after,
                                   hipStream_t stream) {
    if (T <= 0 || n <= 0 || groups <= 0 || n % groups || groups > 65535 || y_stride < n || z_stride < n || out_stride < n)
        return LI_ERR_SIZE;
    if (n / groups <= 256) {
        const long units = (long)T * groups;
        const unsigned blocks = (unsigned)((units + 3) / 4);
        if (out_dtype == LI_F32)
            gated_group_norm_wave_kernel<float><<<blocks, 256, 0, stream>>>(y, y_stride, z, z_stride, w, eps, (float*)out, out_stride, units, groups, n / groups, gate_after);
        else if (out_dtype == LI_BF16)
            gated_group_norm_wave_kernel<bf16_t><<<blocks, 256, 0, stream>>>(y, y_stride, z, z_stride, w, eps, (bf16_t*)out, out_stride, units, groups, n / groups, gate_after);
        else return LI_ERR_DTYPE;
        return li_launch_status();
    }
    const dim3 grid(T, groups);
    if (out_dtype == LI_F32)
        gated_group_norm_kernel<float, 8><<<grid, 256, 0, stream>>>(y, y_stride, z, z_stride, w, eps, (float*)out, out_stride, n / groups, gate_after);
    else if (out_dtype == LI_BF16)
        gated_group_norm_kernel<bf16_t, 8><<<grid, 256, 0, stream>>>(y, y_stride, z, z_stride, w, eps, (bf16_t*)out, out_stride, n / groups, gate_after);
    else return LI_ERR_DTYPE;
    return li_launch_status();
}
