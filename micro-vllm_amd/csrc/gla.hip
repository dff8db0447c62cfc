// Gated linear attention: a memory whose state rows decay one by one, over a ragged step (rows of tokens back to back, as
// in seq_mix.hip).  Per head, with S [n, p] kept per sequence in its state slot:
//   S <- diag(alpha_t) S + k_t v_t^T,   o_t = S^T (q_t * q_scale),   alpha_t = sigmoid(z_t + bias)^(1 / tau)
//   out_t = act( o_t / sqrt(mean(o_t^2) + eps) * w * silu(g_t) )          (norm per head, w shared by the heads)
// One call takes the projections' columns and leaves the operand of the output projection: gates, recurrence, head
// norm and output gate.  All of it in fp32.
//   gla_scan          rows of few tokens: one workgroup per (row, head) with S in registers, token by token
//   gla_chunk_*       rows of many tokens, in chunks of 64.  Within a chunk that starts from state S0, with
//                     G_t = alpha_1 * ... * alpha_t per state row (t counted within the chunk):
//                       O = (G * Q) S0 + B V,  B[t][s] = sum_i q_t[i] k_s[i] (G_t / G_s)[i]  (s <= t)
//                       S_end = diag(G_end) S0 + ((G_end / G) * K)^T V
//     state   per (chunk, head): G_end and what the chunk adds to the state, ((G_end / G) * K)^T V
//     carry   per (row, head, value of the state): the state each chunk starts from, and the one the row leaves
//     out     per (chunk, head): B, O, its norm and gate
// The quotients are never formed: a chunk is four blocks of 16 tokens, G_t / G_s is the product of the gates from the
// start of t's block to t, of whole blocks in between, and from s to the end of s's block - products of numbers in
// (0, 1] that underflow to zero just as the token-by-token run does, whatever the gates are.
#include "recurrence.h"

namespace mv {

constexpr int kGlaMaxN = 512;      // state rows per head
constexpr int kGlaMaxP = 256;      // state columns per head
constexpr int kGCh = 64;
constexpr int kGlaOut = 512;       // threads of the out kernel

struct GlaArgs {
    const float *q, *k, *v, *z, *bias, *gate, *norm;
    int64_t ldq, ldk, ldv, ldz, ldg, ldo;
    float* state;           // [slots, H, n, p]
    void* out;              // [T, ldo] activation type
    const int *row_start, *row_len, *row_ctx, *row_slot;
    int H, n, p, max_len, vec_in, vec_v, vec_out;
    float eps, q_scale, neg_inv_tau;
    // chunks of long rows
    const int *ch_start, *ch_len, *row_ch0, *row_nch;
    float *s0, *gc;         // per (chunk, head): N x P (16 x 16 tiles, a tile's lane (r, g) rows 4 g .. + 3 of column r), N
};

// sigmoid(z + bias)^(1 / tau) = exp(-softplus(-(z + bias)) / tau)
__device__ __forceinline__ float gla_decay(const GlaArgs& a, float z, float bias) {
    return decay_gate(-z, -bias, a.neg_inv_tau);
}

// One workgroup per (head, row).  Thread (ng, cl) holds the state rows ng * R .. + R of column cl; columns are padded to `pw`,
// a power of two, rows to whole threads (their key, query and gate are zero).
template <bool F32, int R>
__global__ void gla_scan_kernel(GlaArgs a, int pw) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x, NT = blockDim.x;
    const int len = a.row_len[b], start = a.row_start[b];
    if (a.max_len > 0 && len > a.max_len) return;      // the chunked form's rows; the whole workgroup
    const int NG = NT / pw, cl = tid & (pw - 1), ng = tid / pw;
    const int n = a.n, p = a.p, rows = NG * R, n0 = ng * R;
    float* qs = lds;
    float* ks = qs + rows;
    float* gs = ks + rows;
    float* pq = gs + rows;          // [NG][pw]
    float* red = pq + NT;           // [pw / 64]
    const bool vc = cl < p;
    float* sp = a.state + (((int64_t)a.row_slot[b] * a.H + h) * n + n0) * p + cl;
    const int mine = vc ? (n - n0 < R ? n - n0 : R) : 0, held = a.row_ctx[b] > 0 ? mine : 0;
    float S[R];
#pragma unroll
    for (int i = 0; i < R; ++i) S[i] = i < held ? sp[(int64_t)i * p] : 0.f;
    const float wn = vc ? a.norm[cl] : 0.f;
    for (int t = 0; t < len; ++t) {
        const int64_t tok = start + t;
        for (int i = tid; i < rows; i += NT) {
            const int64_t c = (int64_t)h * n + i;
            const bool ok = i < n;
            qs[i] = ok ? a.q[tok * a.ldq + c] * a.q_scale : 0.f;
            ks[i] = ok ? a.k[tok * a.ldk + c] : 0.f;
            gs[i] = ok ? gla_decay(a, a.z[tok * a.ldz + c], a.bias ? a.bias[c] : 0.f) : 0.f;
        }
        const float vv = vc ? a.v[tok * a.ldv + (int64_t)h * p + cl] : 0.f;
        const float zz = (vc && ng == 0) ? a.gate[tok * a.ldg + (int64_t)h * p + cl] : 0.f;
        __syncthreads();
        float o = 0.f;
#pragma unroll
        for (int i = 0; i < R; i += 4) {
            const float4 k4 = *reinterpret_cast<const float4*>(ks + n0 + i), g4 = *reinterpret_cast<const float4*>(gs + n0 + i);
            const float4 q4 = *reinterpret_cast<const float4*>(qs + n0 + i);
            S[i] = fmaf(k4.x, vv, g4.x * S[i]);
            S[i + 1] = fmaf(k4.y, vv, g4.y * S[i + 1]);
            S[i + 2] = fmaf(k4.z, vv, g4.z * S[i + 2]);
            S[i + 3] = fmaf(k4.w, vv, g4.w * S[i + 3]);
            o = fmaf(S[i], q4.x, o);
            o = fmaf(S[i + 1], q4.y, o);
            o = fmaf(S[i + 2], q4.z, o);
            o = fmaf(S[i + 3], q4.w, o);
        }
        pq[tid] = o;
        __syncthreads();
        o = 0.f;
        for (int j = 0; j < NG; ++j) o += pq[j * pw + cl];
        // mean square over the head's columns: a wave holds 64 of them (or all of them several times over)
        float ss = o * o;
        for (int m = (pw < 64 ? pw : 64) / 2; m > 0; m >>= 1) ss += __shfl_xor(ss, m, 64);
        if (ng == 0 && (cl & 63) == 0) red[cl >> 6] = ss;
        __syncthreads();
        if (ng == 0 && vc) {
            ss = 0.f;
            for (int j = 0; j < (pw + 63) / 64; ++j) ss += red[j];
            const float inv = 1.0f / sqrtf(ss / (float)p + a.eps);
            ActD<F32>::st((typename ActD<F32>::T*)a.out + tok * a.ldo + (int64_t)h * p + cl,
                          (o * inv) * wn * (zz * sigmoid_d(zz)));
        }
    }
#pragma unroll
    for (int i = 0; i < R; ++i)
        if (i < mine) sp[(int64_t)i * p] = S[i];
}

// One workgroup per (head, chunk).  A wave takes 16 state rows at a time: lane (r, g) holds row r's keys and gates of the
// tokens 4 g .. + 3 of each block of 16, the products of the gates behind a token come from its own four, from the lanes
// with larger g and from the blocks behind, and the weighted keys are the matrix product's operand where they lie; the
// values lie in LDS.
__global__ __launch_bounds__(512) void gla_chunk_state_kernel(GlaArgs a) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int h = blockIdx.x, ch = blockIdx.y, tid = threadIdx.x, NT = blockDim.x;
    const int wv = tid >> 6, lane = tid & 63, r = lane & 15, g = lane >> 4;
    const int n = a.n, p = a.p, N = pad16(n), P = pad16(p), SP = P + 4, nt = N / 16, pt = P / 16;
    const int start = a.ch_start[ch], len = a.ch_len[ch];
    const int64_t unit = (int64_t)ch * a.H + h;
    if (a.vec_v) {
        const int p4 = P / 4;
        for (int i = tid; i < kGCh * p4; i += NT) {
            const int t = i / p4, c = 4 * (i - t * p4);
            float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
            if (t < len && c < p) v = *reinterpret_cast<const float4*>(a.v + (int64_t)(start + t) * a.ldv + (int64_t)h * p + c);
            *reinterpret_cast<float4*>(lds + t * SP + c) = v;
        }
    } else {
        for (int i = tid; i < kGCh * P; i += NT) {
            const int t = i / P, c = i - t * P;
            lds[t * SP + c] = (t < len && c < p) ? a.v[(int64_t)(start + t) * a.ldv + (int64_t)h * p + c] : 0.f;
        }
    }
    float w[4][4], run = 1.f;
    auto keys = [&](int it) {
        const int i = 16 * it + r;
        const int64_t c = (int64_t)h * n + (i < n ? i : n - 1);
        const float bias = a.bias ? a.bias[c] : 0.f;
        float kk[16], zz[16];
#pragma unroll
        for (int e = 0; e < 16; ++e) {
            const int t = 16 * (e >> 2) + 4 * g + (e & 3);
            const int64_t tok = start + (t < len ? t : len - 1);
            kk[e] = a.k[tok * a.ldk + c];
            zz[e] = a.z[tok * a.ldz + c];
        }
        run = 1.f;                           // product of the gates of the blocks behind
#pragma unroll
        for (int blk = 3; blk >= 0; --blk) {
            float al[4], mine = 1.f;
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const bool ok = i < n && 16 * blk + 4 * g + j < len;
                al[j] = ok ? gla_decay(a, zz[4 * blk + j], bias) : 1.f;
                w[blk][j] = ok ? kk[4 * blk + j] : 0.f;
                mine *= al[j];
            }
            const float p1 = __shfl(mine, (lane + 16) & 63, 64), p2 = __shfl(mine, (lane + 32) & 63, 64);
            const float p3 = __shfl(mine, (lane + 48) & 63, 64);
            float suf = run;
            if (g < 3) suf *= p1;
            if (g < 2) suf *= p2;
            if (g < 1) suf *= p3;
#pragma unroll
            for (int j = 3; j >= 0; --j) {
                w[blk][j] *= suf;
                suf *= al[j];
            }
            run *= ((mine * p1) * p2) * p3;
        }
    };
    keys(wv < nt ? wv : 0);
    __syncthreads();
    for (int it = wv; it < nt; it += NT / 64) {
        if (it != wv) keys(it);
        if (g == 0) a.gc[unit * N + 16 * it + r] = run;
        float4* out = reinterpret_cast<float4*>(a.s0 + unit * ((int64_t)N * P)) + it * pt * 64 + lane;
        for (int ct = 0; ct < pt; ++ct) {
            const float* v = lds + 4 * g * SP + 16 * ct + r;
            f32x4_t y0 = f32x4_t{0.f, 0.f, 0.f, 0.f}, y1 = y0;      // neighbouring products do not wait for each other
#pragma unroll
            for (int blk = 0; blk < 4; ++blk) {
                MV_DMFMA(y0, w[blk][0], v[16 * blk * SP]);
                MV_DMFMA(y1, w[blk][1], v[(16 * blk + 1) * SP]);
                MV_DMFMA(y0, w[blk][2], v[(16 * blk + 2) * SP]);
                MV_DMFMA(y1, w[blk][3], v[(16 * blk + 3) * SP]);
            }
            y0 += y1;
            out[ct * 64] = make_float4(y0[0], y0[1], y0[2], y0[3]);
        }
    }
}

// Four state values a thread, in the tiles' order: the state each chunk starts from takes the place of what it adds.
__global__ __launch_bounds__(256) void gla_chunk_carry_kernel(GlaArgs a) {
    const int h = blockIdx.y, b = blockIdx.z, nch = a.row_nch[b], e = blockIdx.x * 256 + threadIdx.x;
    const int n = a.n, p = a.p, N = pad16(n), P = pad16(p), pt = P / 16;
    if (nch == 0 || e >= N * P / 4) return;
    const int tile = e >> 6, it = tile / pt, g = (e >> 4) & 3, row = 16 * it + 4 * g, col = 16 * (tile - it * pt) + (e & 15);
    const bool carried = a.row_ctx[b] > 0;
    float* st = a.state + (((int64_t)a.row_slot[b] * a.H + h) * n + row) * p + col;
    float S[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) S[j] = (carried && col < p && row + j < n) ? st[(int64_t)j * p] : 0.f;
    const int64_t u0 = (int64_t)a.row_ch0[b] * a.H + h;
    constexpr int kB = 4;                    // chunks whose values are requested together
    for (int c0 = 0; c0 < nch; c0 += kB) {
        float4 d[kB], gm[kB];
#pragma unroll
        for (int u = 0; u < kB; ++u) {
            const int64_t unit = u0 + (int64_t)(c0 + u < nch ? c0 + u : nch - 1) * a.H;
            d[u] = reinterpret_cast<const float4*>(a.s0 + unit * ((int64_t)N * P))[e];
            gm[u] = *reinterpret_cast<const float4*>(a.gc + unit * N + row);
        }
#pragma unroll
        for (int u = 0; u < kB; ++u) {
            if (c0 + u >= nch) break;
            const int64_t unit = u0 + (int64_t)(c0 + u) * a.H;
            reinterpret_cast<float4*>(a.s0 + unit * ((int64_t)N * P))[e] = make_float4(S[0], S[1], S[2], S[3]);
            S[0] = fmaf(gm[u].x, S[0], d[u].x);
            S[1] = fmaf(gm[u].y, S[1], d[u].y);
            S[2] = fmaf(gm[u].z, S[2], d[u].z);
            S[3] = fmaf(gm[u].w, S[3], d[u].w);
        }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
        if (col < p && row + j < n) st[(int64_t)j * p] = S[j];
}

// One workgroup per (head, chunk), eight waves.  NM: groups of 32 state rows (n <= 32 NM); CTW: 16-column tiles a wave owns.
// B is kept as ten 16 x 16 tiles (tokens x earlier tokens), in a tile lane (r, g) reads token r, earlier tokens 4 g .. + 3.
template <bool F32, int NM, int CTW>
__global__ __launch_bounds__(kGlaOut, NM <= 4 ? 4 : 2) void gla_chunk_out_kernel(GlaArgs a) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int h = blockIdx.x, ch = blockIdx.y, tid = threadIdx.x;
    const int wv = tid >> 6, lane = tid & 63, r = lane & 15, g = lane >> 4;
    const int n = a.n, p = a.p, N = pad16(n), P = pad16(p), SN = N + 4, nt = N / 16, pt = P / 16;
    float* Q = lds;                    // raw q, then q * (product of the gates from the block's start)
    float* G = Q + kGCh * SN;          // gates, then k * (product of the gates behind the token, in its block)
    float* E = G + kGCh * SN;          // [4][N] products over whole blocks
    float* Bt = E + 4 * N;             // tiles 0..3: diagonal blocks, 4..9: below them
    float* red = Bt + 10 * 256;        // [8][64]
    const int start = a.ch_start[ch], len = a.ch_len[ch];
    const int64_t unit = (int64_t)ch * a.H + h;
    const int blk = wv & 3, half = wv >> 2;
    // this wave's share of the diagonal block `blk`: token 16 blk + r, state rows 16 m + 4 g .. + 3, m = half, half + 2, ..
    float4 kk[NM];
    {
        const int t = 16 * blk + r;
        const float* kp = a.k + (int64_t)(start + (t < len ? t : len - 1)) * a.ldk + (int64_t)h * n;
#pragma unroll
        for (int i = 0; i < NM; ++i) {
            const int c = 16 * (2 * i + half) + 4 * g;
            kk[i] = make_float4(0.f, 0.f, 0.f, 0.f);
            if (t >= len) continue;
            if (a.vec_in) {
                if (c < n) kk[i] = *reinterpret_cast<const float4*>(kp + c);
            } else {
                kk[i].x = c < n ? kp[c] : 0.f;
                kk[i].y = c + 1 < n ? kp[c + 1] : 0.f;
                kk[i].z = c + 2 < n ? kp[c + 2] : 0.f;
                kk[i].w = c + 3 < n ? kp[c + 3] : 0.f;
            }
        }
    }
    const float* bias = a.bias ? a.bias + (int64_t)h * n : nullptr;
    if (a.vec_in) {
        constexpr int kB = 4;          // loads in flight together
        const int n4 = N / 4, real4 = n / 4;
        for (int i0 = tid; i0 < kGCh * n4; i0 += kGlaOut * kB) {
            float4 q_[kB], z_[kB], b_[kB];
#pragma unroll
            for (int u = 0; u < kB; ++u) {
                const int i = i0 + kGlaOut * u, t = i / n4, c = i - t * n4;
                const int64_t tok = start + (t < len ? t : len - 1);
                const int cc = 4 * (c < real4 ? c : real4 - 1);
                q_[u] = *reinterpret_cast<const float4*>(a.q + tok * a.ldq + (int64_t)h * n + cc);
                z_[u] = *reinterpret_cast<const float4*>(a.z + tok * a.ldz + (int64_t)h * n + cc);
                b_[u] = bias ? *reinterpret_cast<const float4*>(bias + cc) : make_float4(0.f, 0.f, 0.f, 0.f);
            }
#pragma unroll
            for (int u = 0; u < kB; ++u) {
                const int i = i0 + kGlaOut * u, t = i / n4, c = i - t * n4;
                if (t >= kGCh) continue;
                const bool ok = t < len && c < real4;
                float4 qv = make_float4(0.f, 0.f, 0.f, 0.f), gv = make_float4(1.f, 1.f, 1.f, 1.f);
                if (ok) {
                    qv = make_float4(q_[u].x * a.q_scale, q_[u].y * a.q_scale, q_[u].z * a.q_scale, q_[u].w * a.q_scale);
                    gv = make_float4(gla_decay(a, z_[u].x, b_[u].x), gla_decay(a, z_[u].y, b_[u].y),
                                     gla_decay(a, z_[u].z, b_[u].z), gla_decay(a, z_[u].w, b_[u].w));
                }
                *reinterpret_cast<float4*>(Q + t * SN + 4 * c) = qv;
                *reinterpret_cast<float4*>(G + t * SN + 4 * c) = gv;
            }
        }
    } else {
        for (int i = tid; i < kGCh * N; i += kGlaOut) {
            const int t = i / N, c = i - t * N;
            const bool ok = t < len && c < n;
            const int64_t tok = start + (t < len ? t : len - 1), cc = (int64_t)h * n + (c < n ? c : n - 1);
            const float qv = a.q[tok * a.ldq + cc], zv = a.z[tok * a.ldz + cc], bv = bias ? bias[c < n ? c : n - 1] : 0.f;
            Q[t * SN + c] = ok ? qv * a.q_scale : 0.f;
            G[t * SN + c] = ok ? gla_decay(a, zv, bv) : 1.f;
        }
    }
    __syncthreads();
    // diagonal blocks: the lane's key walks the tokens behind its own with a running product of gates; what it ends with is
    // the key times the gates to the end of its block
    float sa[16];
#pragma unroll
    for (int t = 0; t < 16; ++t) sa[t] = 0.f;
    {
        const float* l0 = Q + 16 * blk * SN + 4 * g;
        const float* g0 = G + 16 * blk * SN + 4 * g;
#pragma unroll
        for (int i = 0; i < NM; ++i) {
            const int m = 16 * (2 * i + half);
            if (m >= N) continue;
            const float4 own = kk[i];
            float4 w = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
            for (int t = 0; t < 16; ++t) {
                const float4 gt = *reinterpret_cast<const float4*>(g0 + t * SN + m);
                const float4 lt = *reinterpret_cast<const float4*>(l0 + t * SN + m);
                const bool self = t == r;
                w.x = self ? own.x : w.x * gt.x;
                w.y = self ? own.y : w.y * gt.y;
                w.z = self ? own.z : w.z * gt.z;
                w.w = self ? own.w : w.w * gt.w;
                sa[t] = fmaf(lt.x, w.x, fmaf(lt.y, w.y, fmaf(lt.z, w.z, fmaf(lt.w, w.w, sa[t]))));
            }
            kk[i] = w;
        }
    }
    // the lane with (t >> 2) == g keeps token t; both halves of the state rows meet in the tile of the diagonal block
    float dg[4];
#pragma unroll
    for (int t = 0; t < 16; ++t) {
        float x = sa[t];
        x += __shfl_xor(x, 16, 64);
        x += __shfl_xor(x, 32, 64);
        if ((t >> 2) == g) dg[t & 3] = x;
    }
    const int dpos = (r >> 2) * 64 + 16 * g + (r & 3);         // of (token 4 g, earlier token r) in a tile
    if (half == 1)
#pragma unroll
        for (int j = 0; j < 4; ++j) Bt[(4 + blk) * 256 + dpos + 4 * j] = dg[j];     // tiles below the diagonal: free so far
    __syncthreads();
    if (half == 0)
#pragma unroll
        for (int j = 0; j < 4; ++j)
            Bt[blk * 256 + dpos + 4 * j] = r <= 4 * g + j ? dg[j] + Bt[(4 + blk) * 256 + dpos + 4 * j] : 0.f;
    // products of the gates from each block's start: thread per (block, state row)
    for (int i = tid; i < 4 * N; i += kGlaOut) {
        const int b4 = i / N, c = i - b4 * N;
        float* qc = Q + 16 * b4 * SN + c;
        const float* gp = G + 16 * b4 * SN + c;
        float gt[16], qt[16];
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            gt[t] = gp[t * SN];
            qt[t] = qc[t * SN];
        }
        float pre = 1.f;
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            pre *= gt[t];
            qc[t * SN] = qt[t] * pre;
        }
        E[b4 * N + c] = pre;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < NM; ++i) {
        const int m = 16 * (2 * i + half);
        if (m < N) *reinterpret_cast<float4*>(G + (16 * blk + r) * SN + m + 4 * g) = kk[i];
    }
    // the wave's first values and state tile are under way from here on
    float vv[CTW][16];
#pragma unroll
    for (int w = 0; w < CTW; ++w) {
        const int c = 16 * (wv + 8 * w) + r;
        const float* vp = a.v + (int64_t)h * p + (c < p ? c : p - 1);
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const int t = 16 * (i >> 2) + 4 * g + (i & 3);
            vv[w][i] = vp[(int64_t)(start + (t < len ? t : len - 1)) * a.ldv];
        }
    }
    __syncthreads();
    // blocks below the diagonal: B[t][s] for t in block I, s in block J < I, as s x t results (lane (r, g): token r)
    if (wv < 6) {
        const int I = wv == 0 ? 1 : (wv < 3 ? 2 : 3), J = wv == 0 ? 0 : (wv < 3 ? wv - 1 : wv - 3);
        f32x4_t acc = f32x4_t{0.f, 0.f, 0.f, 0.f}, acc2 = acc;
        const float* kr = G + (16 * J + r) * SN + 4 * g;
        const float* qr = Q + (16 * I + r) * SN + 4 * g;
        for (int m = 0; m < N; m += 16) {
            float4 kv = *reinterpret_cast<const float4*>(kr + m);
            const float4 qv = *reinterpret_cast<const float4*>(qr + m);
            for (int M = J + 1; M < I; ++M) {
                const float4 e = *reinterpret_cast<const float4*>(E + M * N + m + 4 * g);
                kv.x *= e.x;
                kv.y *= e.y;
                kv.z *= e.z;
                kv.w *= e.w;
            }
            MV_DMFMA(acc, kv.x, qv.x);
            MV_DMFMA(acc2, kv.y, qv.y);
            MV_DMFMA(acc, kv.z, qv.z);
            MV_DMFMA(acc2, kv.w, qv.w);
        }
        acc += acc2;
        reinterpret_cast<float4*>(Bt)[(4 + wv) * 64 + lane] = make_float4(acc[0], acc[1], acc[2], acc[3]);
    }
    // O, columns x tokens: what the chunk's start contributes
    f32x4_t o[CTW][4];
#pragma unroll
    for (int w = 0; w < CTW; ++w)
#pragma unroll
        for (int I = 0; I < 4; ++I) o[w][I] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const float4* s0 = reinterpret_cast<const float4*>(a.s0 + unit * ((int64_t)N * P)) + lane;
    if (wv < pt) {
        float4 nx[CTW];
#pragma unroll
        for (int w = 0; w < CTW; ++w) nx[w] = s0[(wv + 8 * w < pt ? wv + 8 * w : wv) * 64];
        for (int k = 0; k < nt; ++k) {
            float4 s[CTW], q4[4];
#pragma unroll
            for (int w = 0; w < CTW; ++w) s[w] = nx[w];
            if (k + 1 < nt)
#pragma unroll
                for (int w = 0; w < CTW; ++w) nx[w] = s0[((k + 1) * pt + (wv + 8 * w < pt ? wv + 8 * w : wv)) * 64];
#pragma unroll
            for (int I = 0; I < 4; ++I) q4[I] = *reinterpret_cast<const float4*>(Q + (16 * I + r) * SN + 16 * k + 4 * g);
#pragma unroll
            for (int I = 0; I < 4; ++I) {
#pragma unroll
                for (int w = 0; w < CTW; ++w) {
                    MV_DMFMA(o[w][I], s[w].x, q4[I].x);
                    MV_DMFMA(o[w][I], s[w].y, q4[I].y);
                    MV_DMFMA(o[w][I], s[w].z, q4[I].z);
                    MV_DMFMA(o[w][I], s[w].w, q4[I].w);
                }
                if (I == 3) break;
                const float4 e = *reinterpret_cast<const float4*>(E + I * N + 16 * k + 4 * g);   // decayed over the block
#pragma unroll
                for (int w = 0; w < CTW; ++w) {
                    s[w].x *= e.x;
                    s[w].y *= e.y;
                    s[w].z *= e.z;
                    s[w].w *= e.w;
                }
            }
        }
    }
    __syncthreads();       // all tiles of B are there
    if (wv < pt) {
#pragma unroll
        for (int I = 0; I < 4; ++I)
#pragma unroll
            for (int J = 0; J <= I; ++J) {
                const int tile = I == J ? I : 4 + (I == 1 ? 0 : (I == 2 ? 1 : 3)) + J;
                const float4 bt = reinterpret_cast<const float4*>(Bt)[tile * 64 + lane];
#pragma unroll
                for (int w = 0; w < CTW; ++w) {
                    const bool ok = 16 * (wv + 8 * w) + r < p;
                    MV_DMFMA(o[w][I], ok ? vv[w][4 * J] : 0.f, bt.x);
                    MV_DMFMA(o[w][I], ok ? vv[w][4 * J + 1] : 0.f, bt.y);
                    MV_DMFMA(o[w][I], ok ? vv[w][4 * J + 2] : 0.f, bt.z);
                    MV_DMFMA(o[w][I], ok ? vv[w][4 * J + 3] : 0.f, bt.w);
                }
            }
    }
    // lane (r, g): token 16 I + r, columns 16 ct + 4 g .. + 3.  A tile beyond the head's columns counts for nothing.
#pragma unroll
    for (int I = 0; I < 4; ++I) {
        float ss = 0.f;
#pragma unroll
        for (int w = 0; w < CTW; ++w)
            if (wv + 8 * w < pt) ss += o[w][I][0] * o[w][I][0] + o[w][I][1] * o[w][I][1] + o[w][I][2] * o[w][I][2] + o[w][I][3] * o[w][I][3];
        ss += __shfl_xor(ss, 16, 64);
        ss += __shfl_xor(ss, 32, 64);
        if (g == 0) red[wv * 64 + 16 * I + r] = ss;
    }
    __syncthreads();
#pragma unroll
    for (int I = 0; I < 4; ++I) {
        const int t = 16 * I + r;
        if (t >= len) continue;
        float ss = 0.f;
#pragma unroll
        for (int w = 0; w < 8; ++w) ss += red[w * 64 + t];
        const float inv = 1.0f / sqrtf(ss / (float)p + a.eps);
        const float* gp = a.gate + (int64_t)(start + t) * a.ldg + (int64_t)h * p;
        typename ActD<F32>::T* op = (typename ActD<F32>::T*)a.out + (int64_t)(start + t) * a.ldo + (int64_t)h * p;
#pragma unroll
        for (int w = 0; w < CTW; ++w) {
            if (wv + 8 * w >= pt) continue;
            const int c = 16 * (wv + 8 * w) + 4 * g;
            if (a.vec_out) {       // p a multiple of 16, rows aligned for four values at a time
                const float4 z = *reinterpret_cast<const float4*>(gp + c), nw = *reinterpret_cast<const float4*>(a.norm + c);
                const float4 y = make_float4((o[w][I][0] * inv) * nw.x * (z.x * sigmoid_d(z.x)), (o[w][I][1] * inv) * nw.y * (z.y * sigmoid_d(z.y)),
                                             (o[w][I][2] * inv) * nw.z * (z.z * sigmoid_d(z.z)), (o[w][I][3] * inv) * nw.w * (z.w * sigmoid_d(z.w)));
                if (F32) *reinterpret_cast<float4*>((float*)op + c) = y;
                else *reinterpret_cast<uint2*>((uint16_t*)op + c) = make_uint2(pack_bf16x2(y.x, y.y), pack_bf16x2(y.z, y.w));
            } else {
#pragma unroll
                for (int j = 0; j < 4; ++j)
                    if (c + j < p) ActD<F32>::st(op + c + j, (o[w][I][j] * inv) * a.norm[c + j] * (gp[c + j] * sigmoid_d(gp[c + j])));
            }
        }
    }
}

static size_t gla_out_lds(int n) {
    const int N = (n + 15) & ~15;
    return ((size_t)2 * kGCh * (N + 4) + 4 * N + 10 * 256 + 8 * 64) * sizeof(float);
}

}  // namespace mv

extern "C" {

int mv_gated_linear_chunked_ok(int n, int p) {
    return n > 0 && p > 0 && n <= 256 && p <= mv::kGlaMaxP;
}

int64_t mv_gated_linear_scratch_floats(int n, int p) {
    const int64_t N = (n + 15) & ~15, P = (p + 15) & ~15;
    return N * P + N;
}

int mv_gated_linear_attn(const float* q, int64_t ldq, const float* k, int64_t ldk, const float* v, int64_t ldv,
                         const float* z, int64_t ldz, const float* z_bias, const float* gate, int64_t ldg,
                         const float* norm, float* state, void* out, int64_t ldo, const int32_t* row_start,
                         const int32_t* row_len, const int32_t* row_ctx, const int32_t* row_slot, int rows, int heads,
                         int n, int p, float q_scale, float inv_tau, float eps, float* scratch, const int32_t* ch_start,
                         const int32_t* ch_len, const int32_t* row_ch0, const int32_t* row_nch, int chunks, int max_len,
                         int short_tokens, int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || heads <= 0 || n <= 0 || p <= 0 || chunks < 0) return MV_ERR_INVALID_ARG;
    if (p > kGlaMaxP || n > kGlaMaxN || rows > 65535 || chunks > 65535) return MV_ERR_UNSUPPORTED;
    if (rows == 0) return MV_OK;
    const int64_t hn = (int64_t)heads * n, hp = (int64_t)heads * p;
    if (!q || !k || !v || !z || !gate || !norm || !state || !out || !row_start || !row_len || !row_ctx || !row_slot ||
        ldq < hn || ldk < hn || ldz < hn || ldv < hp || ldg < hp || ldo < hp)
        return MV_ERR_INVALID_ARG;
    if (chunks > 0 && (!scratch || !ch_start || !ch_len || !row_ch0 || !row_nch || max_len <= 0 || !aligned16(scratch)))
        return MV_ERR_INVALID_ARG;
    if (chunks > 0 && !mv_gated_linear_chunked_ok(n, p)) return MV_ERR_UNSUPPORTED;
    GlaArgs a;
    a.q = q; a.k = k; a.v = v; a.z = z; a.bias = z_bias; a.gate = gate; a.norm = norm;
    a.ldq = ldq; a.ldk = ldk; a.ldv = ldv; a.ldz = ldz; a.ldg = ldg; a.ldo = ldo;
    a.state = state; a.out = out;
    a.row_start = row_start; a.row_len = row_len; a.row_ctx = row_ctx; a.row_slot = row_slot;
    a.H = heads; a.n = n; a.p = p; a.max_len = chunks > 0 ? max_len : 0;
    a.eps = eps; a.q_scale = q_scale; a.neg_inv_tau = -inv_tau;
    a.ch_start = ch_start; a.ch_len = ch_len; a.row_ch0 = row_ch0; a.row_nch = row_nch;
    a.vec_in = n % 4 == 0 && ldq % 4 == 0 && ldk % 4 == 0 && ldz % 4 == 0 && aligned16(q) && aligned16(k) && aligned16(z) &&
               (!z_bias || aligned16(z_bias));
    a.vec_v = p % 4 == 0 && ldv % 4 == 0 && aligned16(v);
    a.vec_out = p % 16 == 0 && ldg % 4 == 0 && ldo % 4 == 0 && aligned16(gate) && aligned16(out) && aligned16(norm);
    hipStream_t s = (hipStream_t)stream;
    if (chunks == 0 || short_tokens != 0) {
        int pw = 16;
        while (pw < p) pw *= 2;
        int nt = 256;
        while (nt < 1024 && (int64_t)n * pw > (int64_t)nt * 16) nt *= 2;
        const int ng = nt / pw, npt = (n + ng - 1) / ng;
        const dim3 grid(heads, rows);
#define MV_GLA_SCAN(M_)                                                                                          \
    do {                                                                                                         \
        const size_t lds = ((size_t)3 * ng * M_ + nt + 8) * sizeof(float);                                          \
        if (f32) hipLaunchKernelGGL((gla_scan_kernel<true, M_>), grid, dim3(nt), lds, s, a, pw);                   \
        else hipLaunchKernelGGL((gla_scan_kernel<false, M_>), grid, dim3(nt), lds, s, a, pw);                      \
    } while (0)
        if (npt <= 4) MV_GLA_SCAN(4);
        else if (npt <= 8) MV_GLA_SCAN(8);
        else if (npt <= 16) MV_GLA_SCAN(16);
        else if (npt <= 32) MV_GLA_SCAN(32);
        else if (npt <= 64) MV_GLA_SCAN(64);
        else return MV_ERR_UNSUPPORTED;
#undef MV_GLA_SCAN
    }
    if (chunks > 0) {
        const int64_t N = (n + 15) & ~15, P = (p + 15) & ~15, U = (int64_t)chunks * heads;
        a.s0 = scratch;
        a.gc = a.s0 + U * N * P;
        const size_t lds0 = (size_t)kGCh * (P + 4) * sizeof(float);
        static LdsOptIn opt0;
        if (int rc = ensure_dynamic_lds((const void*)gla_chunk_state_kernel, lds0, opt0)) return rc;
        hipLaunchKernelGGL(gla_chunk_state_kernel, dim3(heads, chunks), dim3(N > 64 ? 512 : 256), lds0, s, a);
        hipLaunchKernelGGL(gla_chunk_carry_kernel, dim3((unsigned)((N * P / 4 + 255) / 256), heads, rows), dim3(256), 0, s, a);
        const size_t lds = gla_out_lds(n);
        static LdsOptIn opt[2][3][2];
        const dim3 go(heads, chunks);
#define MV_GLA_OUT(F32_, NM_, CTW_, I_)                                                                          \
    do {                                                                                                         \
        if (int rc = ensure_dynamic_lds((const void*)gla_chunk_out_kernel<F32_, NM_, CTW_>, lds, opt[F32_][I_][CTW_ - 1])) return rc; \
        hipLaunchKernelGGL((gla_chunk_out_kernel<F32_, NM_, CTW_>), go, dim3(kGlaOut), lds, s, a);                \
    } while (0)
#define MV_GLA_OUT_N(F32_, CTW_)                                                                                 \
    do {                                                                                                         \
        if (N <= 64) MV_GLA_OUT(F32_, 2, CTW_, 0);                                                                \
        else if (N <= 128) MV_GLA_OUT(F32_, 4, CTW_, 1);                                                          \
        else MV_GLA_OUT(F32_, 8, CTW_, 2);                                                                        \
    } while (0)
        if (f32) {
            if (P <= 128) MV_GLA_OUT_N(true, 1); else MV_GLA_OUT_N(true, 2);
        } else {
            if (P <= 128) MV_GLA_OUT_N(false, 1); else MV_GLA_OUT_N(false, 2);
        }
#undef MV_GLA_OUT_N
#undef MV_GLA_OUT
    }
    return check_launch();
}

}  // extern "C"
