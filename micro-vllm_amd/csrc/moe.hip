// Routed feed-forward (mixture of experts) over a step's tokens, everything on the device so that a step
// can be recorded into a graph:
//
//   moe_route    logits = W_router h in fp32 (h in the activation type), the `top` largest (ties: the lower
//                index), weights = softmax over the chosen logits; beside it sigmoid(w_sg . h), the factor
//                of a shared expert (one number per token)
//   moe_route_scored  scores = softmax of the fp32 logits over ALL router outputs; the `top` largest of
//                score + correction are chosen (ties: the lower index), their weights are the scores themselves
//                (without the correction) divided by their sum (+ floor), times `scale`.  Router outputs from
//                `first_pass` on have no expert behind them: they stand for the input itself (moe_combine)
//   moe_route_sigmoid  the `top` largest fp32 logits (ties: the lower index), weights = sigmoid of each chosen
//                logit, not renormalised
//   moe_route_grouped  scores = sigmoid of the fp32 logits; experts come in `groups` equal runs of neighbours, a run is
//                worth the sum of its two largest score + correction, and the `top` largest of score + correction are
//                chosen within the `keep` best runs (ties: the lower index); their weights are the scores themselves
//                (without the correction), not renormalised
//   gated_act_scaled  rows sorted by expert: out = act( f(s g) * (s u) ) with s the weight of the row's (token,
//                choice) pair - an expert that reads weight * h, formed from the products of h itself (the
//                projections are linear)
//   moe_plan     the step's T * top (token, choice) pairs sorted by expert: seg[e] .. seg[e+1] are expert e's
//                rows, order[i] the pair (token * top + choice) in row i, place[pair] its row.  The order inside
//                an expert is whatever the atomics give; no result depends on it, since a row's products do
//                not depend on the other rows (mv_linear_segments)
//   moe_combine  y_t = sum_k weight[t,k] * expert_out[place[t,k]] (+ factor_t * shared_out_t); with a norm given
//                the sum goes through it straight into the stream: y += tanh(alpha sum) w + b.  A choice
//                ids[t,k] >= first_pass adds weight * pass[t] (the feed-forward's own input) instead of an expert's row
// The experts' products themselves are mv_linear_segments (linear_any.hip) with a SiLU-gate between them.
#include "common.h"

namespace mv {

constexpr int kMaxExperts = 1024, kMaxTop = 16;

template <bool F32>
__global__ __launch_bounds__(256) void moe_route_kernel(const void* h_, int64_t ldh, const float* wr, const float* wsg,
                                                        int* ids, float* wts, float* shared_gate, int n, int E,
                                                        int top, int sigmoid_scores) {
    __shared__ float z[kMaxExperts + 1];
    const int t = blockIdx.x, wv = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int units = E + (wsg ? 1 : 0);
    for (int e = wv; e < units; e += 4) {
        const float* w = e < E ? wr + (int64_t)e * n : wsg;
        float dot = 0.f;
        if (F32) {
            const float* h = (const float*)h_ + (int64_t)t * ldh;
#pragma unroll 8
            for (int c = lane; c < n; c += 64) dot = fmaf(h[c], w[c], dot);
        } else {
            const uint16_t* h = (const uint16_t*)h_ + (int64_t)t * ldh;
#pragma unroll 8
            for (int c = lane; c < n; c += 64) dot = fmaf(bf16_bits_to_f32(h[c]), w[c], dot);
        }
        dot = wave_sum(dot);
        if (lane == 0) z[e] = dot;
    }
    __syncthreads();
    if (threadIdx.x == 0) {
        int pick[kMaxTop];
        float val[kMaxTop];
        for (int k = 0; k < top; ++k) {
            int best = -1;
            float bv = -INFINITY;
            for (int e = 0; e < E; ++e) {
                bool taken = false;
                for (int j = 0; j < k; ++j) taken |= pick[j] == e;
                if (!taken && (best < 0 || z[e] > bv)) {
                    best = e;
                    bv = z[e];
                }
            }
            pick[k] = best;
            val[k] = bv;
        }
        float sum = 0.f;
        const float largest = val[0];
        for (int k = 0; k < top; ++k) {
            val[k] = sigmoid_scores ? 1.0f / (1.0f + expf(-val[k])) : expf(val[k] - largest);
            sum += val[k];
        }
        if (sigmoid_scores) sum = 1.0f;      // each chosen expert keeps its own score
        for (int k = 0; k < top; ++k) {
            ids[(int64_t)t * top + k] = pick[k];
            wts[(int64_t)t * top + k] = val[k] / sum;
        }
        if (wsg) shared_gate[t] = 1.0f / (1.0f + expf(-z[E]));
    }
}

template <bool F32>
__global__ __launch_bounds__(256) void moe_route_scored_kernel(const void* h_, int64_t ldh, const float* wr,
                                                               const float* correction, int* ids, float* wts, int n,
                                                               int E, int top, float scale, float floor_) {
    __shared__ float z[kMaxExperts];
    const int t = blockIdx.x, wv = threadIdx.x >> 6, lane = threadIdx.x & 63;
    for (int e = wv; e < E; e += 4) {
        const float* w = wr + (int64_t)e * n;
        float dot = 0.f;
        if (F32) {
            const float* h = (const float*)h_ + (int64_t)t * ldh;
#pragma unroll 8
            for (int c = lane; c < n; c += 64) dot = fmaf(h[c], w[c], dot);
        } else {
            const uint16_t* h = (const uint16_t*)h_ + (int64_t)t * ldh;
#pragma unroll 8
            for (int c = lane; c < n; c += 64) dot = fmaf(bf16_bits_to_f32(h[c]), w[c], dot);
        }
        dot = wave_sum(dot);
        if (lane == 0) z[e] = dot;
    }
    __syncthreads();
    if (threadIdx.x == 0) {
        float largest = z[0], sum = 0.f;
        for (int e = 1; e < E; ++e) largest = fmaxf(largest, z[e]);
        for (int e = 0; e < E; ++e) {
            z[e] = expf(z[e] - largest);
            sum += z[e];
        }
        for (int e = 0; e < E; ++e) z[e] = z[e] / sum;
        int pick[kMaxTop];
        float total = 0.f;
        for (int k = 0; k < top; ++k) {
            int best = -1;
            float bv = -INFINITY;
            for (int e = 0; e < E; ++e) {
                bool taken = false;
                for (int j = 0; j < k; ++j) taken |= pick[j] == e;
                const float c = correction ? z[e] + correction[e] : z[e];
                if (!taken && (best < 0 || c > bv)) {
                    best = e;
                    bv = c;
                }
            }
            pick[k] = best;
            total += z[best];
        }
        total += floor_;
        for (int k = 0; k < top; ++k) {
            ids[(int64_t)t * top + k] = pick[k];
            wts[(int64_t)t * top + k] = (z[pick[k]] / total) * scale;
        }
    }
}

// The group-limited choice of one token, by one wave: sc = scores, ch = choice scores (spoilt), worth = a place per group.
__device__ __forceinline__ void choose_grouped(const float* sc, float* ch, float* worth, int lane, int E, int groups, int keep,
                                               int top, int* ids, float* wts) {
    const int per = E / groups;
    for (int g = lane; g < groups; g += 64) {
        float a = -INFINITY, b = -INFINITY;          // the two largest
        for (int i = 0; i < per; ++i) {
            const float v = ch[g * per + i];
            if (v > a) {
                b = a;
                a = v;
            } else if (v > b) {
                b = v;
            }
        }
        worth[g] = per > 1 ? a + b : a;
    }
    __builtin_amdgcn_wave_barrier();
    // a group that `keep` others are ahead of is out: its experts can no longer be chosen, whatever their scores
    for (int g = lane; g < groups; g += 64) {
        int ahead = 0;
        for (int o = 0; o < groups; ++o) ahead += worth[o] > worth[g] || (worth[o] == worth[g] && o < g);
        if (ahead >= keep)
            for (int i = 0; i < per; ++i) ch[g * per + i] = -INFINITY;
    }
    __builtin_amdgcn_wave_barrier();
    for (int k = 0; k < top; ++k) {
        float bv = -INFINITY;
        int best = E;
        for (int e = lane; e < E; e += 64)
            if (ch[e] > bv) {
                bv = ch[e];
                best = e;
            }
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) {
            const float ov = __shfl_xor(bv, o, 64);
            const int oe = __shfl_xor(best, o, 64);
            if (ov > bv || (ov == bv && oe < best)) {
                bv = ov;
                best = oe;
            }
        }
        best = best < E ? best : E - 1;              // scores that are not numbers choose nothing: stay in bounds
        if (lane == 0) {
            ids[k] = best;
            wts[k] = sc[best];
            ch[best] = -INFINITY;
        }
        __builtin_amdgcn_wave_barrier();
    }
}

// One workgroup per token, a wave per expert in turns.  `vec`: rows in 16-byte pieces (n a multiple of 8, aligned).
template <bool F32>
__global__ __launch_bounds__(1024) void moe_route_grouped_kernel(const void* h_, int64_t ldh, const float* wr,
                                                                 const float* correction, int* ids, float* wts, int n,
                                                                 int E, int groups, int keep, int top, int vec) {
    extern __shared__ float lds[];
    float* sc = lds;                     // scores | choice scores | what each group is worth
    const int t = blockIdx.x, wv = threadIdx.x >> 6, lane = threadIdx.x & 63, NW = blockDim.x >> 6;
    const float* hf = (const float*)h_ + (int64_t)t * ldh;
    const uint16_t* hb = (const uint16_t*)h_ + (int64_t)t * ldh;
    for (int e = wv; e < E; e += NW) {
        const float* w = wr + (int64_t)e * n;
        float dot = 0.f;
        if (vec) {
#pragma unroll 2
            for (int c = 8 * lane; c < n; c += 512) {
                const float4 wa = *reinterpret_cast<const float4*>(w + c), wb = *reinterpret_cast<const float4*>(w + c + 4);
                float x[8];
                if (F32) {
                    const float4 a = *reinterpret_cast<const float4*>(hf + c), b = *reinterpret_cast<const float4*>(hf + c + 4);
                    x[0] = a.x; x[1] = a.y; x[2] = a.z; x[3] = a.w; x[4] = b.x; x[5] = b.y; x[6] = b.z; x[7] = b.w;
                } else {
                    const uint4 a = ld16(hb + c);
                    x[0] = bf16_lo(a.x); x[1] = bf16_hi(a.x); x[2] = bf16_lo(a.y); x[3] = bf16_hi(a.y);
                    x[4] = bf16_lo(a.z); x[5] = bf16_hi(a.z); x[6] = bf16_lo(a.w); x[7] = bf16_hi(a.w);
                }
                dot = fmaf(x[0], wa.x, fmaf(x[1], wa.y, fmaf(x[2], wa.z, fmaf(x[3], wa.w, dot))));
                dot = fmaf(x[4], wb.x, fmaf(x[5], wb.y, fmaf(x[6], wb.z, fmaf(x[7], wb.w, dot))));
            }
        } else {
            for (int c = lane; c < n; c += 64) dot = fmaf(F32 ? hf[c] : bf16_bits_to_f32(hb[c]), w[c], dot);
        }
        dot = wave_sum(dot);
        if (lane == 0) {
            const float s = 1.0f / (1.0f + expf(-dot));
            sc[e] = s;
            sc[E + e] = correction ? s + correction[e] : s;
        }
    }
    __syncthreads();
    if (wv == 0)
        choose_grouped(sc, sc + E, sc + 2 * E, lane, E, groups, keep, top, ids + (int64_t)t * top, wts + (int64_t)t * top);
}

// The same for steps of many tokens: a workgroup per 16 tokens, the logits as 16 experts x 16 tokens on
// v_mfma_f32_16x16x4_f32 (true fp32), eight waves sharing the contraction.  n a multiple of 16, rows aligned for pieces of
// four values, E <= kRouteTileE.
constexpr int kRouteTileE = 256;

template <bool F32>
__global__ __launch_bounds__(512) void moe_route_grouped_tile_kernel(const void* h_, int64_t ldh, const float* wr,
                                                                     const float* correction, int* ids, float* wts, int T,
                                                                     int n, int E, int groups, int keep, int top) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    float* part = lds;                   // [8 waves][16 tokens][16 experts]
    float* sc = lds + 8 * 256;           // [16 tokens][scores | choice scores | what each group is worth]
    const int per_tok = 2 * E + groups;
    const int t0 = blockIdx.x * 16, wv = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane & 15, g = lane >> 4;
    const int tn = T - t0 < 16 ? T - t0 : 16;
    const int64_t row = (int64_t)(t0 + (r < tn ? r : 0)) * ldh;
    const float* hf = (const float*)h_ + row;
    const uint16_t* hb = (const uint16_t*)h_ + row;
    for (int e0 = 0; e0 < E; e0 += 16) {
        const float* w = wr + (int64_t)(e0 + r < E ? e0 + r : e0) * n;
        f32x4_t a0 = f32x4_t{0.f, 0.f, 0.f, 0.f}, a1 = a0;
#pragma unroll 4
        for (int c = 16 * wv + 4 * g; c < n; c += 128) {
            const float4 wc = *reinterpret_cast<const float4*>(w + c);
            float4 x;
            if (F32) {
                x = *reinterpret_cast<const float4*>(hf + c);
            } else {
                const uint2 b = *reinterpret_cast<const uint2*>(hb + c);
                x = make_float4(bf16_lo(b.x), bf16_hi(b.x), bf16_lo(b.y), bf16_hi(b.y));
            }
            a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(wc.x, x.x, a0, 0, 0, 0);
            a1 = __builtin_amdgcn_mfma_f32_16x16x4f32(wc.y, x.y, a1, 0, 0, 0);
            a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(wc.z, x.z, a0, 0, 0, 0);
            a1 = __builtin_amdgcn_mfma_f32_16x16x4f32(wc.w, x.w, a1, 0, 0, 0);
        }
        a0 += a1;                        // lane (r, g): experts e0 + 4 g .. + 3 of token r
        *reinterpret_cast<float4*>(part + wv * 256 + r * 16 + 4 * g) = make_float4(a0[0], a0[1], a0[2], a0[3]);
        __syncthreads();
        if (threadIdx.x < 256) {
            float z = 0.f;
#pragma unroll
            for (int i = 0; i < 8; ++i) z += part[i * 256 + threadIdx.x];
            const int e = e0 + (threadIdx.x & 15);
            if (e < E) {
                float* s = sc + (threadIdx.x >> 4) * per_tok;
                const float v = 1.0f / (1.0f + expf(-z));
                s[e] = v;
                s[E + e] = correction ? v + correction[e] : v;
            }
        }
        __syncthreads();
    }
    for (int u = wv; u < tn; u += 8) {
        float* s = sc + u * per_tok;
        choose_grouped(s, s + E, s + 2 * E, lane, E, groups, keep, top, ids + (int64_t)(t0 + u) * top, wts + (int64_t)(t0 + u) * top);
    }
}

__global__ __launch_bounds__(1024) void moe_plan_kernel(const int* ids, int* seg, int* order, int* place, int pairs,
                                                        int E) {
    __shared__ int cnt[kMaxExperts + 1];
    __shared__ int cur[kMaxExperts];
    for (int e = threadIdx.x; e <= E; e += 1024) cnt[e] = 0;
    __syncthreads();
    for (int i = threadIdx.x; i < pairs; i += 1024) atomicAdd(&cnt[ids[i]], 1);
    __syncthreads();
    if (threadIdx.x == 0) {
        int run = 0;
        for (int e = 0; e < E; ++e) {
            const int c = cnt[e];
            cur[e] = run;
            seg[e] = run;
            run += c;
        }
        seg[E] = run;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < pairs; i += 1024) {
        const int row = atomicAdd(&cur[ids[i]], 1);
        order[row] = i;
        place[i] = row;
    }
}

// norm_w != NULL: the sum does not go to y but through the norm after the sublayer into the stream,
// x += tanh(alpha sum) w + b, and h (optional) = x in the activation type
template <bool F32>
__global__ __launch_bounds__(256) void moe_combine_kernel(const float* eo, int64_t lde, const int* place,
                                                          const float* wts, const float* so, int64_t lds_,
                                                          const float* shared_gate, float* y, int64_t ldy, int n,
                                                          int top, const float* norm_w, const float* norm_b,
                                                          const float* norm_alpha, void* h_, int64_t ldh,
                                                          const int* ids, int first_pass, const void* pass_,
                                                          int64_t ldp) {
    const int t = blockIdx.x;
    int rows[kMaxTop];
    float w[kMaxTop];
    for (int k = 0; k < top; ++k) {
        rows[k] = place[(int64_t)t * top + k];
        w[k] = wts ? wts[(int64_t)t * top + k] : 1.0f;
        if (ids && ids[(int64_t)t * top + k] >= first_pass) rows[k] = -1;   // the input itself, not an expert's row
    }
    const float g = so ? (shared_gate ? shared_gate[t] : 1.0f) : 0.f;
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c < n) {
        float acc = 0.f;
        for (int k = 0; k < top; ++k) {
            float v;
            if (rows[k] >= 0) v = eo[(int64_t)rows[k] * lde + c];
            else if (F32) v = ((const float*)pass_)[(int64_t)t * ldp + c];
            else v = bf16_bits_to_f32(((const uint16_t*)pass_)[(int64_t)t * ldp + c]);
            acc = fmaf(w[k], v, acc);
        }
        if (so) acc = fmaf(g, so[(int64_t)t * lds_ + c], acc);
        if (norm_w) {
            acc = y[(int64_t)t * ldy + c] + fmaf(tanhf(norm_alpha[0] * acc), norm_w[c], norm_b[c]);
            if (h_) {
                if (F32) ((float*)h_)[(int64_t)t * ldh + c] = acc;
                else ((uint16_t*)h_)[(int64_t)t * ldh + c] = (uint16_t)f32_to_bf16_bits(acc);
            }
        }
        y[(int64_t)t * ldy + c] = acc;
    }
}

template <bool F32>
__global__ __launch_bounds__(256) void gated_act_scaled_kernel(const float* a, int64_t lda, void* out_, int64_t ldo,
                                                               int n, int kind, float limit, float slope,
                                                               const float* scale, const int* order) {
    const int64_t row = blockIdx.x;
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c >= n) return;
    const float sc = scale[order ? order[row] : row];
    const float v = gated_act_f(sc * a[row * lda + c], sc * a[row * lda + n + c], kind, limit, slope);
    if (F32) ((float*)out_)[row * ldo + c] = v;
    else ((uint16_t*)out_)[row * ldo + c] = (uint16_t)f32_to_bf16_bits(v);
}

}  // namespace mv

extern "C" {

int mv_moe_route(const void* h, int64_t ldh, const float* w_router, const float* w_shared_gate, int32_t* ids,
                 float* weights, float* shared_gate, int tokens, int n, int experts, int top, int f32,
                 mv_stream_t stream) {
    using namespace mv;
    if (tokens < 0 || n <= 0 || experts <= 0 || experts > kMaxExperts || top <= 0 || top > kMaxTop || top > experts)
        return MV_ERR_INVALID_ARG;
    if (tokens == 0) return MV_OK;
    if (!h || !w_router || !ids || !weights || (w_shared_gate && !shared_gate) || ldh < n) return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    if (f32) hipLaunchKernelGGL(moe_route_kernel<true>, dim3(tokens), dim3(256), 0, s, h, ldh, w_router, w_shared_gate, ids, weights, shared_gate, n, experts, top, 0);
    else hipLaunchKernelGGL(moe_route_kernel<false>, dim3(tokens), dim3(256), 0, s, h, ldh, w_router, w_shared_gate, ids, weights, shared_gate, n, experts, top, 0);
    return check_launch();
}

int mv_moe_route_scored(const void* h, int64_t ldh, const float* w_router, const float* correction, int32_t* ids,
                        float* weights, int tokens, int n, int experts, int top, float scale, float sum_floor, int f32,
                        mv_stream_t stream) {
    using namespace mv;
    if (tokens < 0 || n <= 0 || experts <= 0 || experts > kMaxExperts || top <= 0 || top > kMaxTop || top > experts)
        return MV_ERR_INVALID_ARG;
    if (tokens == 0) return MV_OK;
    if (!h || !w_router || !ids || !weights || ldh < n) return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    if (f32) hipLaunchKernelGGL(moe_route_scored_kernel<true>, dim3(tokens), dim3(256), 0, s, h, ldh, w_router, correction, ids, weights, n, experts, top, scale, sum_floor);
    else hipLaunchKernelGGL(moe_route_scored_kernel<false>, dim3(tokens), dim3(256), 0, s, h, ldh, w_router, correction, ids, weights, n, experts, top, scale, sum_floor);
    return check_launch();
}

int mv_moe_route_sigmoid(const void* h, int64_t ldh, const float* w_router, int32_t* ids, float* weights, int tokens,
                         int n, int experts, int top, int f32, mv_stream_t stream) {
    using namespace mv;
    if (tokens < 0 || n <= 0 || experts <= 0 || experts > kMaxExperts || top <= 0 || top > kMaxTop || top > experts)
        return MV_ERR_INVALID_ARG;
    if (tokens == 0) return MV_OK;
    if (!h || !w_router || !ids || !weights || ldh < n) return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    if (f32) hipLaunchKernelGGL(moe_route_kernel<true>, dim3(tokens), dim3(256), 0, s, h, ldh, w_router, (const float*)nullptr, ids, weights, (float*)nullptr, n, experts, top, 1);
    else hipLaunchKernelGGL(moe_route_kernel<false>, dim3(tokens), dim3(256), 0, s, h, ldh, w_router, (const float*)nullptr, ids, weights, (float*)nullptr, n, experts, top, 1);
    return check_launch();
}

int mv_moe_route_grouped(const void* h, int64_t ldh, const float* w_router, const float* correction, int32_t* ids,
                         float* weights, int tokens, int n, int experts, int groups, int keep, int top, int f32,
                         mv_stream_t stream) {
    using namespace mv;
    if (tokens < 0 || n <= 0 || experts <= 0 || experts > kMaxExperts || top <= 0 || top > kMaxTop || groups <= 0 ||
        experts % groups || keep <= 0 || keep > groups || top > keep * (experts / groups))
        return MV_ERR_INVALID_ARG;
    if (tokens == 0) return MV_OK;
    if (!h || !w_router || !ids || !weights || ldh < n) return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    if (tokens > 64 && experts <= kRouteTileE && n % 16 == 0 && ldh % 4 == 0 && aligned16(h) && aligned16(w_router)) {
        const size_t lds = (8 * 256 + (size_t)16 * (2 * experts + groups)) * sizeof(float);
        const dim3 tiles((tokens + 15) / 16);
        if (f32) hipLaunchKernelGGL(moe_route_grouped_tile_kernel<true>, tiles, dim3(512), lds, s, h, ldh, w_router, correction, ids, weights, tokens, n, experts, groups, keep, top);
        else hipLaunchKernelGGL(moe_route_grouped_tile_kernel<false>, tiles, dim3(512), lds, s, h, ldh, w_router, correction, ids, weights, tokens, n, experts, groups, keep, top);
        return check_launch();
    }
    const int vec = n % 8 == 0 && ldh % 8 == 0 && aligned16(h) && aligned16(w_router);
    int nt = 256;
    while (nt < 1024 && nt / 64 < experts) nt *= 2;
    const size_t lds = (size_t)(2 * experts + groups) * sizeof(float);
    if (f32) hipLaunchKernelGGL(moe_route_grouped_kernel<true>, dim3(tokens), dim3(nt), lds, s, h, ldh, w_router, correction, ids, weights, n, experts, groups, keep, top, vec);
    else hipLaunchKernelGGL(moe_route_grouped_kernel<false>, dim3(tokens), dim3(nt), lds, s, h, ldh, w_router, correction, ids, weights, n, experts, groups, keep, top, vec);
    return check_launch();
}

int mv_gated_act_scaled(const float* a, int64_t lda, void* out, int64_t ldo, int rows, int n, int kind, float limit,
                        float slope, const float* scale, const int32_t* order, int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0 || kind < 0 || kind > 2) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!a || !out || !scale || lda < 2 * (int64_t)n || ldo < n) return MV_ERR_INVALID_ARG;
    const dim3 grid(rows, (n + 255) / 256);
    hipStream_t s = (hipStream_t)stream;
    if (f32) hipLaunchKernelGGL(gated_act_scaled_kernel<true>, grid, dim3(256), 0, s, a, lda, out, ldo, n, kind, limit, slope, scale, order);
    else hipLaunchKernelGGL(gated_act_scaled_kernel<false>, grid, dim3(256), 0, s, a, lda, out, ldo, n, kind, limit, slope, scale, order);
    return check_launch();
}

int mv_moe_plan(const int32_t* ids, int32_t* seg, int32_t* order, int32_t* place, int pairs, int experts,
                mv_stream_t stream) {
    using namespace mv;
    if (pairs < 0 || experts <= 0 || experts > kMaxExperts) return MV_ERR_INVALID_ARG;
    if (!ids || !seg || !order || !place) return MV_ERR_INVALID_ARG;
    hipLaunchKernelGGL(moe_plan_kernel, dim3(1), dim3(1024), 0, (hipStream_t)stream, ids, seg, order, place, pairs,
                       experts);
    return check_launch();
}

int mv_moe_combine(const float* expert_out, int64_t lde, const int32_t* place, const float* weights,
                   const float* shared_out, int64_t lds, const float* shared_gate, float* y, int64_t ldy,
                   const float* norm_w, const float* norm_b, const float* norm_alpha, void* h, int64_t ldh, int tokens,
                   int n, int top, int f32, const int32_t* ids, int first_pass, const void* pass, int64_t ldp,
                   mv_stream_t stream) {
    using namespace mv;
    if (tokens < 0 || n <= 0 || top <= 0 || top > kMaxTop) return MV_ERR_INVALID_ARG;
    if (tokens == 0) return MV_OK;
    if (!expert_out || !place || !y || lde < n || ldy < n ||
        (shared_out && lds < n))
        return MV_ERR_INVALID_ARG;
    if (norm_w ? (!norm_b || !norm_alpha || (h && ldh < n)) : h != nullptr) return MV_ERR_INVALID_ARG;
    if (ids && (!pass || ldp < n || first_pass < 0)) return MV_ERR_INVALID_ARG;
    const dim3 grid(tokens, (n + 255) / 256);
    if (f32) hipLaunchKernelGGL(moe_combine_kernel<true>, grid, dim3(256), 0, (hipStream_t)stream, expert_out, lde, place, weights, shared_out, lds, shared_gate, y, ldy, n, top, norm_w, norm_b, norm_alpha, h, ldh, ids, first_pass, pass, ldp);
    else hipLaunchKernelGGL(moe_combine_kernel<false>, grid, dim3(256), 0, (hipStream_t)stream, expert_out, lde, place, weights, shared_out, lds, shared_gate, y, ldy, n, top, norm_w, norm_b, norm_alpha, h, ldh, ids, first_pass, pass, ldp);
    return check_launch();
}

}  // extern "C"
