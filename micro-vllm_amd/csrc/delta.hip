// Delta-rule memory with a decay per state row, over a ragged step (rows of tokens back to back, as in seq_mix.hip).
// Per head, with S [n, p] kept per sequence in its state slot:
//   S <- diag(g_t) S;   u_t = beta_t (v_t - S^T k_t);   S <- S + k_t u_t^T;   o_t = S^T q_t
// g_t in (0, 1)^n, q and k unit vectors that a group of heads may share.
//
//   delta_prep     the short convolutions with SiLU over the q | k | v columns of one projection, unit length per
//                  head of q and k, beta = sigmoid, and the low-rank inputs of the gates in the activation type
//   delta_rule     rows of few tokens: one workgroup per (row, head) with S in registers, token by token; rows of
//                  many tokens: chunks of 64 (below).  Both form the gates g = exp(-exp(A) softplus(a + bias)) and
//                  hand out act( o / rms(o) * w * sigmoid(z) )
// All of it in fp32; only what goes to a projection is of the activation type.
#include "recurrence.h"

namespace mv {

struct DeltaRows {
    const int *tok_row, *row_start, *row_len, *row_ctx, *row_slot;
};

constexpr int kDeltaMaxTaps = 16;
constexpr int kDeltaMaxN = 512;     // state rows per head

struct DeltaPrepArgs {
    const float* proj;      // [T, ldp]: q [K n] | k [K n] | v [H p] at 0, beta logits at b_off, low-rank columns at low_off
    int64_t ldp, ldo, ldl;
    int b_off, low_off, low_n;
    float* state;           // [slots, taps - 1, C]
    const float* wt;        // [taps, C]
    float* out;             // [T, C]
    float* beta;            // [T, H]
    void* low;              // [T, low_n] activation type
    DeltaRows r;
    int T, K, n, H, p, taps, in_place;
    float eps, qscale;
};

// One wave per (token, unit): a head of q, a head of k, 256 channels of v, or the betas with the low-rank columns.
// in_place: every row has one token, so the wave that reads a channel's kept inputs also moves them on.
template <bool F32>
__global__ __launch_bounds__(256) void delta_prep_kernel(DeltaPrepArgs a) {
    const int lane = threadIdx.x & 63;
    const int vu = (a.H * a.p + 255) / 256, units = 2 * a.K + vu + 1;
    const int unit = blockIdx.y;                                    // the four waves of a workgroup: neighbouring tokens
    const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (t >= a.T) return;
    const float* row = a.proj + (int64_t)t * a.ldp;
    if (unit == units - 1) {
        for (int h = lane; h < a.H; h += 64) a.beta[(int64_t)t * a.H + h] = sigmoid_d(row[a.b_off + h]);
        typename ActD<F32>::T* lo = (typename ActD<F32>::T*)a.low + (int64_t)t * a.ldl;
        for (int c = lane; c < a.low_n; c += 64) ActD<F32>::st(lo + c, row[a.low_off + c]);
        return;
    }
    const bool head = unit < 2 * a.K;
    const int C = 2 * a.K * a.n + a.H * a.p;
    const int c0 = head ? unit * a.n : 2 * a.K * a.n + (unit - 2 * a.K) * 256;
    const int cnt = head ? a.n : (C - c0 < 256 ? C - c0 : 256);
    const int b = a.r.tok_row[t], rel = t - a.r.row_start[b], keep = a.taps - 1;
    const bool carried = a.r.row_ctx[b] > 0;
    float* st = a.state + (int64_t)a.r.row_slot[b] * keep * C;
    float y[kDeltaMaxN / 64];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < kDeltaMaxN / 64; ++i) {
        y[i] = 0.f;
        if (64 * i >= cnt) continue;
        const int cl = lane + 64 * i;
        if (cl >= cnt) continue;
        const int c = c0 + cl;
        float acc = 0.f;
        for (int j = 0; j < a.taps; ++j) {
            const int src = rel - keep + j;
            float v;
            if (src >= 0) v = row[(int64_t)(j - keep) * a.ldp + c];
            else v = carried ? st[(int64_t)(src + keep) * C + c] : 0.f;
            acc = fmaf(a.wt[(int64_t)j * C + c], v, acc);
            // the channel's kept inputs move on by one (tap j of this token is tap j - 1 of the next)
            if (a.in_place && j > 0) st[(int64_t)(j - 1) * C + c] = v;
        }
        y[i] = acc * sigmoid_d(acc);
        ss += y[i] * y[i];
    }
    float f = 1.0f;
    if (head) f = (1.0f / sqrtf(wave_sum(ss) + a.eps)) * (unit < a.K ? a.qscale : 1.0f);
#pragma unroll
    for (int i = 0; i < kDeltaMaxN / 64; ++i) {
        const int cl = lane + 64 * i;
        if (cl < cnt) a.out[(int64_t)t * a.ldo + c0 + cl] = y[i] * f;
    }
}

// The same for up to four taps: a wave takes TB neighbouring tokens of its unit and keeps their inputs in registers, so
// that a token's row is read once instead of once per tap; NI: 64-channel groups of a unit (a head, or a stretch of v).
template <bool F32, int NI, int TB>
__global__ __launch_bounds__(256) void delta_prep4_kernel(DeltaPrepArgs a) {
    const int lane = threadIdx.x & 63, unit = blockIdx.y;
    const int vu = (a.H * a.p + 64 * NI - 1) / (64 * NI), units = 2 * a.K + vu + 1;
    const int t0 = (blockIdx.x * 4 + (threadIdx.x >> 6)) * TB;
    if (t0 >= a.T) return;
    const int tn = a.T - t0 < TB ? a.T - t0 : TB;
    if (unit == units - 1) {
        for (int tb = 0; tb < tn; ++tb) {
            const int64_t t = t0 + tb;
            const float* row = a.proj + t * a.ldp;
            for (int h = lane; h < a.H; h += 64) a.beta[t * a.H + h] = sigmoid_d(row[a.b_off + h]);
            typename ActD<F32>::T* lo = (typename ActD<F32>::T*)a.low + t * a.ldl;
            for (int c = lane; c < a.low_n; c += 64) ActD<F32>::st(lo + c, row[a.low_off + c]);
        }
        return;
    }
    const bool head = unit < 2 * a.K;
    const int C = 2 * a.K * a.n + a.H * a.p;
    const int c0 = head ? unit * a.n : 2 * a.K * a.n + (unit - 2 * a.K) * 64 * NI;
    const int cnt = head ? a.n : (C - c0 < 64 * NI ? C - c0 : 64 * NI);
    const int keep = a.taps - 1, skip = 4 - a.taps;
    float w[NI][4], x[NI][TB + 3];
#pragma unroll
    for (int i = 0; i < NI; ++i) {
        const int cl = lane + 64 * i;
        const bool ok = cl < cnt;
        const float* col = a.proj + c0 + (ok ? cl : 0);
#pragma unroll
        for (int s = 0; s < TB + 3; ++s) {
            const int ft = t0 - 3 + s;
            x[i][s] = (ok && ft >= 0 && ft < a.T) ? col[(int64_t)ft * a.ldp] : 0.f;
        }
#pragma unroll
        for (int j = 0; j < 4; ++j) w[i][j] = (ok && j >= skip) ? a.wt[(int64_t)(j - skip) * C + c0 + cl] : 0.f;
    }
    int row[TB], at[TB];          // each token's row and its place there, looked up together
#pragma unroll
    for (int tb = 0; tb < TB; ++tb) row[tb] = a.r.tok_row[tb < tn ? t0 + tb : t0];
#pragma unroll
    for (int tb = 0; tb < TB; ++tb) at[tb] = t0 + tb - a.r.row_start[row[tb]];
#pragma unroll
    for (int tb = 0; tb < TB; ++tb) {
        if (tb >= tn) break;
        const int t = t0 + tb, b = row[tb], rel = at[tb];
        float y[NI], ss = 0.f;
        if (rel >= 3 && !a.in_place) {
#pragma unroll
            for (int i = 0; i < NI; ++i) {
                float acc = 0.f;
#pragma unroll
                for (int j = 0; j < 4; ++j) acc = fmaf(w[i][j], x[i][tb + j], acc);
                y[i] = acc;
            }
        } else {
            // the row's first tokens: inputs from before the step lie in the slot
            const bool carried = a.r.row_ctx[b] > 0;
            float* st = a.state + (int64_t)a.r.row_slot[b] * keep * C + c0;
            float v[NI][4];
#pragma unroll
            for (int i = 0; i < NI; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    const int src = rel - 3 + j, cl = lane + 64 * i;
                    v[i][j] = x[i][tb + j];
                    if (src < 0) v[i][j] = (carried && j >= skip && cl < cnt) ? st[(int64_t)(src + keep) * C + cl] : 0.f;
                }
#pragma unroll
            for (int i = 0; i < NI; ++i) {
                float acc = 0.f;
#pragma unroll
                for (int j = 0; j < 4; ++j) acc = fmaf(w[i][j], v[i][j], acc);
                y[i] = acc;
                if (a.in_place && lane + 64 * i < cnt)
#pragma unroll
                    for (int j = 1; j < 4; ++j)
                        if (j > skip) st[(int64_t)(j - skip - 1) * C + lane + 64 * i] = v[i][j];
            }
        }
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            y[i] *= sigmoid_d(y[i]);
            ss += y[i] * y[i];
        }
        float f = 1.0f;
        if (head) f = (1.0f / sqrtf(wave_sum(ss) + a.eps)) * (unit < a.K ? a.qscale : 1.0f);
#pragma unroll
        for (int i = 0; i < NI; ++i)
            if (lane + 64 * i < cnt) a.out[(int64_t)t * a.ldo + c0 + lane + 64 * i] = y[i] * f;
    }
}

// keeps each row's last taps - 1 inputs (rows of any length; used when some row has more than one token)
__global__ __launch_bounds__(256) void delta_conv_state_kernel(DeltaPrepArgs a, int B) {
    const int C = 2 * a.K * a.n + a.H * a.p, keep = a.taps - 1;
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= (int64_t)B * C) return;
    const int b = (int)(i / C), c = (int)(i % C);
    const int len = a.r.row_len[b], start = a.r.row_start[b];
    const bool carried = a.r.row_ctx[b] > 0;
    float* st = a.state + (int64_t)a.r.row_slot[b] * keep * C + c;
    float old[kDeltaMaxTaps];
    for (int s = 0; s < keep; ++s) old[s] = carried ? st[(int64_t)s * C] : 0.f;
    for (int s = 0; s < keep; ++s) {
        const int rel = len - keep + s;
        st[(int64_t)s * C] = rel >= 0 ? a.proj[(int64_t)(start + rel) * a.ldp + c] : old[s + len];
    }
}

struct DeltaArgs {
    const float* qkv;       // [T, ldq]: q [K n] | k [K n] | v [H p], as delta_prep leaves them
    const float* a;         // [T, lda]: raw gate inputs [H n]
    const float* z;         // [T, ldz]: logits of the output gate [H p]
    const float *beta, *dt_bias, *a_log, *norm;
    int64_t ldq, lda, ldz, ldo;
    float* state;           // [slots, H, n, p]
    void* out;              // [T, ldo] activation type
    DeltaRows r;
    int K, H, n, p, max_len, vec;
    float eps;
    // chunks of long rows
    const int *ch_start, *ch_len, *row_ch0, *row_nch;
    float *qd, *wk, *kt, *uv, *bm, *s0, *gc;     // scratch, see DeltaScratch
};

// One workgroup per (head, row).  Thread (ng, cl) holds the state rows ng * npt .. + npt of column cl; columns are
// padded to `pw`, a power of two.  The two sums over state rows (what the key reads, what the query reads) are formed in one
// pass over the decayed state; the write's share of the read-out is u (k . q).
template <bool F32, int MAXN>
__global__ void delta_scan_kernel(DeltaArgs a, int pw) {
    extern __shared__ float lds[];
    const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x, NT = blockDim.x;
    const int len = a.r.row_len[b], start = a.r.row_start[b];
    if (a.max_len > 0 && len > a.max_len) return;      // the chunked form's rows; the whole workgroup
    const int NG = NT / pw, cl = tid & (pw - 1), ng = tid / pw;
    const int n = a.n, p = a.p, npt = (n + NG - 1) / NG, n0 = ng * npt;
    float* qs = lds;
    float* ks = qs + n;
    float* gs = ks + n;
    float* pk = gs + n;             // [NG][pw]
    float* pq = pk + NT;            // [NG][pw]
    float* pd = pq + NT;            // [NG] partial sums of k . q
    float* red = pd + NG;           // [pw / 64]
    const bool vc = cl < p;
    const int kh = h / (a.H / a.K);
    const bool carried = a.r.row_ctx[b] > 0;
    float* sp = a.state + (((int64_t)a.r.row_slot[b] * a.H + h) * n + n0) * p + cl;
    float S[MAXN];
#pragma unroll
    for (int i = 0; i < MAXN; ++i) S[i] = (carried && vc && i < npt && n0 + i < n) ? sp[(int64_t)i * p] : 0.f;
    const float neg_a = -expf(a.a_log[h]);
    const float wn = vc ? a.norm[cl] : 0.f;
    for (int t = 0; t < len; ++t) {
        const int64_t tok = start + t;
        const float* qp = a.qkv + tok * a.ldq + (int64_t)kh * n;
        const float* kp = qp + (int64_t)a.K * n;
        for (int i = tid; i < n; i += NT) {
            qs[i] = qp[i];
            ks[i] = kp[i];
            gs[i] = decay_gate(a.a[tok * a.lda + (int64_t)h * n + i], a.dt_bias[(int64_t)h * n + i], neg_a);
        }
        const float vv = vc ? a.qkv[tok * a.ldq + (int64_t)2 * a.K * n + (int64_t)h * p + cl] : 0.f;
        const float zz = (vc && ng == 0) ? a.z[tok * a.ldz + (int64_t)h * p + cl] : 0.f;
        const float bt = a.beta[tok * a.H + h];
        __syncthreads();
        float rk = 0.f, rq = 0.f, kq = 0.f;
#pragma unroll
        for (int i = 0; i < MAXN; ++i) {
            if (i < npt && n0 + i < n) {
                const float k_ = ks[n0 + i], q_ = qs[n0 + i];
                S[i] *= gs[n0 + i];
                rk = fmaf(S[i], k_, rk);
                rq = fmaf(S[i], q_, rq);
                kq = fmaf(k_, q_, kq);
            }
        }
        pk[tid] = rk;
        pq[tid] = rq;
        if (cl == 0) pd[ng] = kq;
        __syncthreads();
        rk = rq = kq = 0.f;
        for (int j = 0; j < NG; ++j) {
            rk += pk[j * pw + cl];
            rq += pq[j * pw + cl];
            kq += pd[j];
        }
        const float u = bt * (vv - rk);
        const float o = vc ? fmaf(u, kq, rq) : 0.f;
#pragma unroll
        for (int i = 0; i < MAXN; ++i)
            if (i < npt && n0 + i < n) S[i] = fmaf(ks[n0 + i], u, S[i]);
        // mean square over the head's columns: a wave holds 64 of them (or all of them several times over)
        float ss = o * o;
        for (int m = (pw < 64 ? pw : 64) / 2; m > 0; m >>= 1) ss += __shfl_xor(ss, m, 64);
        if (ng == 0 && (cl & 63) == 0) red[cl >> 6] = ss;
        __syncthreads();
        if (ng == 0 && vc) {
            ss = 0.f;
            for (int j = 0; j < (pw + 63) / 64; ++j) ss += red[j];
            const float inv = 1.0f / sqrtf(ss / (float)p + a.eps);
            ActD<F32>::st((typename ActD<F32>::T*)a.out + tok * a.ldo + (int64_t)h * p + cl, (o * inv) * wn * sigmoid_d(zz));
        }
    }
    if (vc) {
#pragma unroll
        for (int i = 0; i < MAXN; ++i)
            if (i < npt && n0 + i < n) sp[(int64_t)i * p] = S[i];
    }
}

// ---- the same recurrence in chunks of 64 tokens, for long rows -------------------------------------------------
// Within a chunk that starts from state S0, G_t = g_1 * ... * g_t per state row (t counted within the chunk):
//   A[t][s] = sum_i k_t[i] k_s[i] (G_t / G_s)[i]  (s < t),   B[t][s] = the same with q_t  (s <= t)
//   (I + diag(beta) A) U = diag(beta) (V - (G * K) S0)        row by row: U = Uv - Wk S0
//   O = (G * Q) S0 + B U,      S_end = diag(G_end) S0 + sum_s ((G_end / G_s) * k_s) u_s^T
//   intra   per (chunk, head): A and B, the unit triangular system solved for Uv and Wk, and the operands G * Q,
//           (G_end / G) * K (transposed) and G_end
//   carry   per (row, head, 16 columns): U and the state from chunk to chunk
//   inter   per (chunk, head): O, its unit-RMS, weight and sigmoid gate
// The quotients are never formed.  A chunk is cut into four blocks of 16 tokens; G_t / G_s is the product of the gates
// from the start of t's block to t, of whole blocks in between, and from s to the end of s's block - products of
// numbers in (0, 1) that underflow to zero just as the token-by-token run does, whatever the gates are.  Within a
// block a lane walks the tokens t after its s with a running product.  Matrix products are v_mfma_f32_16x16x4_f32
// (true fp32): operand A lane (r, g) = A[r][g], B lane (r, g) = B[g][r], result lane (r, g) = C[4 g + j][r]
// (r = lane % 16, g = lane / 16).  The contraction index is a label: in step j of a group of 16, slot g stands for
// index 4 g + j, so a result can be the next product's operand B where it lies and operand A is a 16-byte read.
constexpr int kDCh = 64;

// scratch per (chunk, head): qd, wk (64 x n16) and kt (n16 x 64) in the order in which the lanes of a wave read them as
// operand A - tile by tile of 16 x 16, lane (r, g) holding row r, columns 4 g .. + 3 -, uv (64 x p16) and s0 (n16 x p16)
// as slabs of 16 columns, bm [64][64], gc [n16]
constexpr int kIntra = 512;      // threads of the intra kernel: two waves a SIMD, one workgroup a compute unit

__global__ __launch_bounds__(kIntra) void delta_chunk_intra_kernel(DeltaArgs a) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int ch = blockIdx.y, h = blockIdx.x, tid = threadIdx.x;
    const int wv = tid >> 6, lane = tid & 63, r = lane & 15, g = lane >> 4;
    const int n = a.n, p = a.p, N = pad16(n), P = pad16(p), SN = N + 4;
    float* Q = lds;                      // raw q, then q * (product of the gates from the block's start)
    float* Kp = Q + kDCh * SN;           // raw k, then the same for k
    float* Gn = Kp + kDCh * SN;          // gates, then k * (product of the gates behind the token, in its block)
    float* Am = Gn + kDCh * SN;          // -beta A [64][68]
    float* Di = Am + kDCh * 68;          // [4][16][20] inverses of the diagonal blocks of I + beta A
    float* E = Di + 4 * 16 * 20;         // [4][N] products over whole blocks
    float* bs = E + 4 * N;               // [64]
    const int start = a.ch_start[ch], len = a.ch_len[ch], kh = h / (a.H / a.K);
    const int64_t unit = (int64_t)ch * a.H + h;
    const float neg_a = -expf(a.a_log[h]);
    constexpr int kB = 8;            // loads in flight together (addresses clamped, values selected afterwards)
    for (int i0 = tid; i0 < kDCh * N; i0 += kIntra * kB) {
        float q_[kB], k_[kB], a_[kB], b_[kB];
#pragma unroll
        for (int u = 0; u < kB; ++u) {
            const int i = i0 + kIntra * u, t = i / N, c = i - t * N;
            const int64_t tok = start + (t < len ? t : len - 1);
            const int cc = c < n ? c : n - 1;
            const float* qp = a.qkv + tok * a.ldq + (int64_t)kh * n + cc;
            q_[u] = qp[0];
            k_[u] = qp[(int64_t)a.K * n];
            a_[u] = a.a[tok * a.lda + (int64_t)h * n + cc];
            b_[u] = a.dt_bias[(int64_t)h * n + cc];
        }
#pragma unroll
        for (int u = 0; u < kB; ++u) {
            const int i = i0 + kIntra * u, t = i / N, c = i - t * N;
            if (t >= kDCh) continue;
            const bool ok = t < len && c < n;
            Q[t * SN + c] = ok ? q_[u] : 0.f;
            Kp[t * SN + c] = ok ? k_[u] : 0.f;
            Gn[t * SN + c] = ok ? decay_gate(a_[u], b_[u], neg_a) : 1.f;
        }
    }
    if (tid < kDCh) bs[tid] = tid < len ? a.beta[(int64_t)(start + tid) * a.H + h] : 0.f;
    __syncthreads();
    // diagonal blocks, A by the first four waves and B by the others: lane (r, g) holds column s = r, state rows
    // 16 m + 4 g .. + 3
    {
        const int blk = wv & 3;
        const bool isb = wv >= 4;
        float sa[16];
#pragma unroll
        for (int t = 0; t < 16; ++t) sa[t] = 0.f;
        const float* l0 = (isb ? Q : Kp) + 16 * blk * SN + 4 * g;
        const float* k0 = Kp + 16 * blk * SN + 4 * g;
        const float* g0 = Gn + 16 * blk * SN + 4 * g;
        for (int m = 0; m < N; m += 16) {
            const float4 ks = *reinterpret_cast<const float4*>(k0 + r * SN + m);
            float4 w = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
            for (int t = 0; t < 16; ++t) {
                const float4 gt = *reinterpret_cast<const float4*>(g0 + t * SN + m);
                const float4 lt = *reinterpret_cast<const float4*>(l0 + t * SN + m);
                const bool self = t == r;
                w.x = self ? ks.x : w.x * gt.x;
                w.y = self ? ks.y : w.y * gt.y;
                w.z = self ? ks.z : w.z * gt.z;
                w.w = self ? ks.w : w.w * gt.w;
                sa[t] = fmaf(lt.x, w.x, fmaf(lt.y, w.y, fmaf(lt.z, w.z, fmaf(lt.w, w.w, sa[t]))));
            }
        }
        float* bm = a.bm + unit * (kDCh * kDCh);
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            float x = sa[t];
            x += __shfl_xor(x, 16, 64);
            x += __shfl_xor(x, 32, 64);
            if ((t >> 2) == g) {
                const int tt = 16 * blk + t;
                if (isb) bm[tt * kDCh + 16 * blk + r] = r <= t ? x : 0.f;
                else Am[tt * 68 + 16 * blk + r] = r < t ? -bs[tt] * x : 0.f;
            }
        }
    }
    __syncthreads();
    // products of the gates, in place: thread per (block, state row)
    for (int i = tid; i < 4 * N; i += kIntra) {
        const int blk = i / N, c = i - blk * N;
        float* qc = Q + 16 * blk * SN + c;
        float* kc = Kp + 16 * blk * SN + c;
        float* gc = Gn + 16 * blk * SN + c;
        float gt[16], kk[16];
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            gt[t] = gc[t * SN];
            kk[t] = kc[t * SN];
        }
        float suf = 1.f;
#pragma unroll
        for (int t = 15; t >= 0; --t) {
            gc[t * SN] = kk[t] * suf;
            suf *= gt[t];
        }
        float pre = 1.f;
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            pre *= gt[t];
            kc[t * SN] = kk[t] * pre;
            qc[t * SN] *= pre;
        }
        E[blk * N + c] = pre;
    }
    // inverses of the unit triangular diagonal blocks: lane r owns column r, forward substitution
    if (wv < 4 && g == 0) {
        float x[16];
        const float* m = Am + (16 * wv) * 68 + 16 * wv;
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            float s = t == r ? 1.f : 0.f;
#pragma unroll
            for (int j = 0; j < t; ++j) s = fmaf(m[t * 68 + j], x[j], s);
            x[t] = s;
            Di[(wv * 16 + t) * 20 + r] = s;
        }
    }
    __syncthreads();
    // blocks below the diagonal: six block pairs, A and B each
    for (int id = wv; id < 12; id += kIntra / 64) {
        const int pair = id >> 1;
        const bool isb = id & 1;
        const int I = pair == 0 ? 1 : (pair < 3 ? 2 : 3), J = pair == 0 ? 0 : (pair < 3 ? pair - 1 : pair - 3);
        f32x4_t acc = f32x4_t{0.f, 0.f, 0.f, 0.f};
        const float* ar = (isb ? Q : Kp) + (16 * I + r) * SN + 4 * g;
        const float* br = Gn + (16 * J + r) * SN + 4 * g;
        for (int m = 0; m < N; m += 16) {
            const float4 av = *reinterpret_cast<const float4*>(ar + m);
            float4 bv = *reinterpret_cast<const float4*>(br + m);
            for (int M = J + 1; M < I; ++M) {
                const float4 e = *reinterpret_cast<const float4*>(E + M * N + m + 4 * g);
                bv.x *= e.x;
                bv.y *= e.y;
                bv.z *= e.z;
                bv.w *= e.w;
            }
            MV_DMFMA(acc, av.x, bv.x);
            MV_DMFMA(acc, av.y, bv.y);
            MV_DMFMA(acc, av.z, bv.z);
            MV_DMFMA(acc, av.w, bv.w);
        }
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int t = 16 * I + 4 * g + j, s = 16 * J + r;
            if (isb) a.bm[unit * (kDCh * kDCh) + t * kDCh + s] = acc[j];
            else Am[t * 68 + s] = -bs[t] * acc[j];
        }
    }
    // the wave's first 16 columns of V are under way from here on
    float vv[16];
    auto load_v = [&](int tile) {
        const int c = 16 * tile + r < p ? 16 * tile + r : p - 1;
        const float* vp = a.qkv + (int64_t)2 * a.K * n + (int64_t)h * p + c;
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const int t = 16 * (i >> 2) + 4 * g + (i & 3);
            vv[i] = vp[(int64_t)(start + (t < len ? t : len - 1)) * a.ldq];
        }
    };
    if (wv < P / 16) load_v(wv);
    // operands of the other two kernels, 16 x 16 tiles in operand order
    const int nt = N / 16;
    float4* qd = reinterpret_cast<float4*>(a.qd + unit * (kDCh * N));
    float4* kt = reinterpret_cast<float4*>(a.kt + unit * (kDCh * N));
    for (int i = tid; i < 16 * N; i += kIntra) {
        const int rr = i & 15, gg = (i >> 4) & 3, tl = i >> 6;
        {
            const int blk = tl / nt, c = 16 * (tl - blk * nt) + 4 * gg;
            float4 v = *reinterpret_cast<const float4*>(Q + (16 * blk + rr) * SN + c);
            for (int M = 0; M < blk; ++M) {
                const float4 e = *reinterpret_cast<const float4*>(E + M * N + c);
                v.x *= e.x;
                v.y *= e.y;
                v.z *= e.z;
                v.w *= e.w;
            }
            qd[i] = v;
        }
        {
            const int blk = tl & 3, c = 16 * (tl >> 2) + rr;
            const float* k4 = Gn + (16 * blk + 4 * gg) * SN + c;
            float f = 1.f;
            for (int M = blk + 1; M < 4; ++M) f *= E[M * N + c];
            kt[i] = make_float4(k4[0] * f, k4[SN] * f, k4[2 * SN] * f, k4[3 * SN] * f);
        }
    }
    for (int c = tid; c < N; c += kIntra) a.gc[unit * N + c] = ((E[c] * E[N + c]) * E[2 * N + c]) * E[3 * N + c];
    __syncthreads();
    // the triangular system, 16 columns at a time: first those of V, then those of G * K
    const int pt = P / 16, ntile = pt + N / 16;
    float* uv = a.uv + unit * (kDCh * P);
    for (int tile = wv; tile < ntile; tile += kIntra / 64) {
        const bool isv = tile < pt;
        const int c = 16 * (isv ? tile : tile - pt) + r;
        if (isv && tile != wv) load_v(tile);
        f32x4_t X[4];
        float e = 1.f;           // product of the blocks before I for column c of G * K
#pragma unroll
        for (int I = 0; I < 4; ++I) {
            f32x4_t acc;
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int t = 16 * I + 4 * g + j;
                float v;
                if (isv) v = (t < len && c < p) ? vv[4 * I + j] : 0.f;
                else v = Kp[t * SN + c] * e;
                acc[j] = bs[t] * v;
            }
            if (!isv) e *= E[I * N + c];
#pragma unroll
            for (int J = 0; J < I; ++J) {
                const float4 m = *reinterpret_cast<const float4*>(Am + (16 * I + r) * 68 + 16 * J + 4 * g);
                MV_DMFMA(acc, m.x, X[J][0]);
                MV_DMFMA(acc, m.y, X[J][1]);
                MV_DMFMA(acc, m.z, X[J][2]);
                MV_DMFMA(acc, m.w, X[J][3]);
            }
            const float4 d = *reinterpret_cast<const float4*>(Di + (16 * I + r) * 20 + 4 * g);
            X[I] = f32x4_t{0.f, 0.f, 0.f, 0.f};
            MV_DMFMA(X[I], d.x, acc[0]);
            MV_DMFMA(X[I], d.y, acc[1]);
            MV_DMFMA(X[I], d.z, acc[2]);
            MV_DMFMA(X[I], d.w, acc[3]);
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int t = 16 * I + 4 * g + j;
                if (isv) uv[(tile * kDCh + t) * 16 + r] = X[I][j];
                else Q[t * SN + c] = X[I][j];          // q is not needed any more
            }
        }
    }
    __syncthreads();
    float4* wk = reinterpret_cast<float4*>(a.wk + unit * (kDCh * N));
    for (int i = tid; i < 16 * N; i += kIntra) {
        const int rr = i & 15, gg = (i >> 4) & 3, tl = i >> 6, blk = tl / nt;
        wk[i] = *reinterpret_cast<const float4*>(Q + (16 * blk + rr) * SN + 16 * (tl - blk * nt) + 4 * gg);
    }
}

// One workgroup per (head, 16 state columns, row).  Wave w forms U for the tokens 16 w .. + 15 of a chunk and owns the
// state rows of the 16-row tiles w, w + 4, ...; the state (as operand) and U pass through LDS.  NT: 16-row tiles; FULL: the state has exactly NT of them (no tests between the products).
template <int NT, bool FULL>
__global__ __launch_bounds__(256) void delta_chunk_carry_kernel(DeltaArgs a) {
    constexpr int OWN = (NT + 3) / 4;
    __shared__ float Ss[NT * 16][20];
    __shared__ float Us[kDCh][20];
    const int h = blockIdx.x, c0 = blockIdx.y * 16, b = blockIdx.z;
    const int nch = a.row_nch[b];
    if (nch == 0) return;
    const int tid = threadIdx.x, wv = tid >> 6, lane = tid & 63, r = lane & 15, g = lane >> 4;
    const int n = a.n, p = a.p, N = pad16(n), P = pad16(p), nt = N / 16;
    const bool carried = a.r.row_ctx[b] > 0;
    float* st = a.state + ((int64_t)a.r.row_slot[b] * a.H + h) * n * p + c0 + r;
    const bool vc = c0 + r < p;
    f32x4_t S[OWN];
#pragma unroll
    for (int o = 0; o < OWN; ++o) {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int i = 16 * (wv + 4 * o) + 4 * g + j;
            S[o][j] = (carried && vc && i < n) ? st[(int64_t)i * p] : 0.f;
            if (i < NT * 16) Ss[i][r] = S[o][j];
        }
    }
    const int64_t u0 = (int64_t)a.row_ch0[b] * a.H + h;
    struct Operands {
        float4 wk[NT], kt[OWN][4], gm[OWN];
        f32x4_t uv;
    };
    auto fetch = [&](int64_t unit, Operands& x) {
        const float4* w = reinterpret_cast<const float4*>(a.wk + unit * (kDCh * N)) + wv * nt * 64 + lane;
#pragma unroll
        for (int i = 0; i < NT; ++i)
            if (FULL || i < nt) x.wk[i] = w[64 * i];
#pragma unroll
        for (int o = 0; o < OWN; ++o) {
            const int it = wv + 4 * o;
            if (it < nt || (FULL && NT % 4 == 0)) {
                const float4* k = reinterpret_cast<const float4*>(a.kt + unit * (kDCh * N)) + it * 256 + lane;
#pragma unroll
                for (int t = 0; t < 4; ++t) x.kt[o][t] = k[64 * t];
                x.gm[o] = *reinterpret_cast<const float4*>(a.gc + unit * N + 16 * it + 4 * g);
            }
        }
        const float* up = a.uv + unit * (kDCh * P) + (c0 / 16) * (kDCh * 16) + (16 * wv + 4 * g) * 16 + r;
#pragma unroll
        for (int j = 0; j < 4; ++j) x.uv[j] = up[j * 16];
    };
    // three sets of operands: a chunk's are requested while the two before it are worked on
    auto body = [&](Operands& cur, int c) {
        const int64_t unit = u0 + (int64_t)c * a.H;
        // two accumulators: neighbouring products do not wait for each other
        f32x4_t w0 = f32x4_t{0.f, 0.f, 0.f, 0.f}, w1 = w0;
#pragma unroll
        for (int i = 0; i < NT; ++i) {
            if (FULL || i < nt) {
                const int k = 16 * i + 4 * g;
                MV_DMFMA(w0, cur.wk[i].x, Ss[k][r]);
                MV_DMFMA(w1, cur.wk[i].y, Ss[k + 1][r]);
                MV_DMFMA(w0, cur.wk[i].z, Ss[k + 2][r]);
                MV_DMFMA(w1, cur.wk[i].w, Ss[k + 3][r]);
            }
        }
        float* up = a.uv + unit * (kDCh * P) + (c0 / 16) * (kDCh * 16) + (16 * wv + 4 * g) * 16 + r;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const float u = cur.uv[j] - (w0[j] + w1[j]);
            Us[16 * wv + 4 * g + j][r] = u;
            up[j * 16] = u;
        }
        float* sp = a.s0 + unit * ((int64_t)N * P) + (c0 / 16) * (N * 16) + r;
#pragma unroll
        for (int o = 0; o < OWN; ++o) {
            const int it = wv + 4 * o;
            if (it < nt || (FULL && NT % 4 == 0)) {
#pragma unroll
                for (int j = 0; j < 4; ++j) sp[(16 * it + 4 * g + j) * 16] = S[o][j];    // what this chunk starts from
            }
        }
        __syncthreads();
#pragma unroll
        for (int o = 0; o < OWN; ++o) {
            const int it = wv + 4 * o;
            if (it >= nt && !(FULL && NT % 4 == 0)) continue;
            f32x4_t y0 = f32x4_t{S[o][0] * cur.gm[o].x, S[o][1] * cur.gm[o].y, S[o][2] * cur.gm[o].z, S[o][3] * cur.gm[o].w};
            f32x4_t y1 = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int t = 0; t < 4; ++t) {
                const int k = 16 * t + 4 * g;
                MV_DMFMA(y0, cur.kt[o][t].x, Us[k][r]);
                MV_DMFMA(y1, cur.kt[o][t].y, Us[k + 1][r]);
                MV_DMFMA(y0, cur.kt[o][t].z, Us[k + 2][r]);
                MV_DMFMA(y1, cur.kt[o][t].w, Us[k + 3][r]);
            }
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                S[o][j] = y0[j] + y1[j];
                Ss[16 * it + 4 * g + j][r] = S[o][j];
            }
        }
        if (c + 3 < nch) fetch(unit + 3 * (int64_t)a.H, cur);
        __syncthreads();
    };
    Operands x0, x1, x2;
    fetch(u0, x0);
    if (nch > 1) fetch(u0 + a.H, x1);
    if (nch > 2) fetch(u0 + 2 * (int64_t)a.H, x2);
    __syncthreads();
    for (int c = 0; c < nch; c += 3) {
        body(x0, c);
        if (c + 1 < nch) body(x1, c + 1);
        if (c + 2 < nch) body(x2, c + 2);
    }
#pragma unroll
    for (int o = 0; o < OWN; ++o)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int i = 16 * (wv + 4 * o) + 4 * g + j;
            if (vc && i < n) st[(int64_t)i * p] = S[o][j];
        }
}

// One workgroup per (head, chunk), 16 tokens a wave: lane (r, g) ends with token r, columns 16 ct + 4 g .. + 3.
// FULL: exactly PT tiles of 16 columns (no tests between the products).
template <int PT, bool FULL>
__device__ __forceinline__ void load_slabs(f32x4_t (&x)[PT], const float* src, int64_t slab, int pt) {
#pragma unroll
    for (int ct = 0; ct < PT; ++ct)
        if (FULL || ct < pt) x[ct] = *reinterpret_cast<const f32x4_t*>(src + ct * slab);
}

template <bool F32, int PT, bool FULL>
__global__ __launch_bounds__(256) void delta_chunk_inter_kernel(DeltaArgs a) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int h = blockIdx.x, ch = blockIdx.y, tid = threadIdx.x;
    const int wv = tid >> 6, lane = tid & 63, r = lane & 15, g = lane >> 4;
    const int p = a.p, N = pad16(a.n), P = pad16(p), pt = P / 16, SP = P + 4;
    const int64_t unit = (int64_t)ch * a.H + h;
    const int start = a.ch_start[ch], len = a.ch_len[ch];
    f32x4_t o[PT];
#pragma unroll
    for (int ct = 0; ct < PT; ++ct) o[ct] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const float4* qd = reinterpret_cast<const float4*>(a.qd + unit * (kDCh * N)) + wv * (N / 16) * 64 + lane;
    const float* bm = a.bm + unit * (kDCh * kDCh) + (16 * wv + r) * kDCh + 4 * g;
    const float* s0 = a.s0 + unit * ((int64_t)N * P);
    const float* uv = a.uv + unit * (kDCh * P);
    // 64 rows of the right-hand operand at a time - the state's, then U's - through LDS, the next ones in registers
    // while these are used.  Slabs of 16 columns: thread (tid / 4, tid % 4) moves one 16-byte piece of a row per slab.
    const int stages = (N + kDCh - 1) / kDCh + 1, sr = tid >> 2, sc = 4 * (tid & 3);
    f32x4_t nx[PT], nw[4];        // the next stage's rows, and the wave's left-hand operand for them
    const int nt = N / 16;
#pragma unroll
    for (int k = 0; k < 4; ++k) nw[k] = *reinterpret_cast<const f32x4_t*>(qd + (k < nt ? k : nt - 1) * 64);
    load_slabs<PT, FULL>(nx, s0 + (sr < N ? sr : N - 1) * 16 + sc, (int64_t)N * 16, pt);
    for (int stage = 0; stage < stages; ++stage) {
        const bool isu = stage == stages - 1;
        const int k0 = stage * kDCh;
        __syncthreads();
#pragma unroll
        for (int ct = 0; ct < PT; ++ct)
            if (FULL || ct < pt) *reinterpret_cast<f32x4_t*>(lds + sr * SP + 16 * ct + sc) = nx[ct];
        f32x4_t w[4];
#pragma unroll
        for (int k = 0; k < 4; ++k) w[k] = nw[k];
        __syncthreads();
        if (!isu) {
            const bool nu = stage + 1 == stages - 1;
            const int n0 = k0 + kDCh, rows = nu ? kDCh : N - n0;
            load_slabs<PT, FULL>(nx, (nu ? uv : s0 + n0 * 16) + (sr < rows ? sr : rows - 1) * 16 + sc, (int64_t)(nu ? kDCh : N) * 16, pt);
#pragma unroll
            for (int k = 0; k < 4; ++k) {
                const int i = n0 / 16 + k;
                nw[k] = nu ? *reinterpret_cast<const f32x4_t*>(bm + 16 * k) : *reinterpret_cast<const f32x4_t*>(qd + (i < nt ? i : nt - 1) * 64);
            }
        }
        // of the state what is left, of U no tokens behind the wave's own
        const int top = isu ? 16 * (wv + 1) : (N - k0 < kDCh ? N - k0 : kDCh);
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            if (16 * k >= top) break;
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const float* s = lds + (16 * k + 4 * g + j) * SP + r;
#pragma unroll
                for (int ct = 0; ct < PT; ++ct)
                    if (FULL || ct < pt) MV_DMFMA(o[ct], s[16 * ct], w[k][j]);
            }
        }
    }
    float ss = 0.f;
#pragma unroll
    for (int ct = 0; ct < PT; ++ct)
        if (FULL || ct < pt) ss += o[ct][0] * o[ct][0] + o[ct][1] * o[ct][1] + o[ct][2] * o[ct][2] + o[ct][3] * o[ct][3];
    ss += __shfl_xor(ss, 16, 64);
    ss += __shfl_xor(ss, 32, 64);
    const int t = 16 * wv + r;
    if (t >= len) return;
    const float inv = 1.0f / sqrtf(ss / (float)p + a.eps);
    const float* zp = a.z + (int64_t)(start + t) * a.ldz + (int64_t)h * p;
    typename ActD<F32>::T* op = (typename ActD<F32>::T*)a.out + (int64_t)(start + t) * a.ldo + (int64_t)h * p;
#pragma unroll
    for (int ct = 0; ct < PT; ++ct) {
        if (!FULL && ct >= pt) continue;
        if (a.vec) {        // p a multiple of 16, rows aligned for four values at a time
            const int c = 16 * ct + 4 * g;
            const float4 z = *reinterpret_cast<const float4*>(zp + c), w = *reinterpret_cast<const float4*>(a.norm + c);
            const float4 y = make_float4((o[ct][0] * inv) * w.x * sigmoid_d(z.x), (o[ct][1] * inv) * w.y * sigmoid_d(z.y),
                                         (o[ct][2] * inv) * w.z * sigmoid_d(z.z), (o[ct][3] * inv) * w.w * sigmoid_d(z.w));
            if (F32) *reinterpret_cast<float4*>((float*)op + c) = y;
            else *reinterpret_cast<uint2*>((uint16_t*)op + c) = make_uint2(pack_bf16x2(y.x, y.y), pack_bf16x2(y.z, y.w));
            continue;
        }
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int c = 16 * ct + 4 * g + j;
            if (c < p) ActD<F32>::st(op + c, (o[ct][j] * inv) * a.norm[c] * sigmoid_d(zp[c]));
        }
    }
}

static size_t delta_intra_lds(int n) {
    const int N = (n + 15) & ~15;
    return ((size_t)3 * kDCh * (N + 4) + kDCh * 68 + 4 * 16 * 20 + 4 * N + kDCh) * sizeof(float);
}

}  // namespace mv

extern "C" {

int mv_delta_prep(const float* proj, int64_t ldp, int b_off, int low_off, int low_n, float* state, const float* wt,
                  float* out, int64_t ldo, float* beta, void* low, int64_t ldl, const int32_t* tok_row,
                  const int32_t* row_start, const int32_t* row_len, const int32_t* row_ctx, const int32_t* row_slot,
                  int tokens, int rows, int kv_heads, int n, int heads, int p, int taps, float eps, float q_scale,
                  int f32, mv_stream_t stream) {
    using namespace mv;
    if (tokens < 0 || rows < 0 || kv_heads <= 0 || heads <= 0 || heads % kv_heads || n <= 0 || p <= 0 || taps < 1 ||
        taps > kDeltaMaxTaps || low_n < 0)
        return MV_ERR_INVALID_ARG;
    if (n > kDeltaMaxN) return MV_ERR_UNSUPPORTED;
    if (tokens == 0) return MV_OK;
    const int C = 2 * kv_heads * n + heads * p;
    if (!proj || (taps > 1 && !state) || !wt || !out || !beta || (low_n > 0 && !low) || !tok_row || !row_start ||
        !row_len || !row_ctx || !row_slot || ldp < C || ldo < C || b_off < C || ldp < b_off + heads ||
        (low_n > 0 && (low_off < C || ldp < low_off + low_n || ldl < low_n)))
        return MV_ERR_INVALID_ARG;
    DeltaPrepArgs a;
    a.proj = proj; a.ldp = ldp; a.ldo = ldo; a.ldl = ldl; a.b_off = b_off; a.low_off = low_off; a.low_n = low_n;
    a.state = state; a.wt = wt; a.out = out; a.beta = beta; a.low = low;
    a.r = DeltaRows{tok_row, row_start, row_len, row_ctx, row_slot};
    a.T = tokens; a.K = kv_heads; a.n = n; a.H = heads; a.p = p; a.taps = taps;
    a.in_place = tokens == rows && taps > 1;       // every row has one token
    a.eps = eps; a.qscale = q_scale;
    hipStream_t s = (hipStream_t)stream;
    const int ni = n <= 64 ? 1 : n <= 128 ? 2 : n <= 256 ? 4 : 8;
    const int vw = taps <= 4 ? 64 * ni : 256;
    const int units = 2 * kv_heads + (heads * p + vw - 1) / vw + 1;
    if (units > 65535) return MV_ERR_UNSUPPORTED;
    if (taps <= 4) {
        const int tb = tokens > 64 ? 4 : 1;
        const dim3 grid((tokens + 4 * tb - 1) / (4 * tb), units);
#define MV_PREP4(NI_)                                                                                                  \
    do {                                                                                                               \
        if (f32 && tb == 4) hipLaunchKernelGGL((delta_prep4_kernel<true, NI_, 4>), grid, dim3(256), 0, s, a);            \
        else if (f32) hipLaunchKernelGGL((delta_prep4_kernel<true, NI_, 1>), grid, dim3(256), 0, s, a);                  \
        else if (tb == 4) hipLaunchKernelGGL((delta_prep4_kernel<false, NI_, 4>), grid, dim3(256), 0, s, a);             \
        else hipLaunchKernelGGL((delta_prep4_kernel<false, NI_, 1>), grid, dim3(256), 0, s, a);                          \
    } while (0)
        if (ni == 1) MV_PREP4(1); else if (ni == 2) MV_PREP4(2); else if (ni == 4) MV_PREP4(4); else MV_PREP4(8);
#undef MV_PREP4
    } else {
        const dim3 grid((tokens + 3) / 4, units);
        if (f32) hipLaunchKernelGGL(delta_prep_kernel<true>, grid, dim3(256), 0, s, a);
        else hipLaunchKernelGGL(delta_prep_kernel<false>, grid, dim3(256), 0, s, a);
    }
    if (taps > 1 && !a.in_place) {
        const int64_t work = (int64_t)rows * C;
        hipLaunchKernelGGL(delta_conv_state_kernel, dim3((unsigned)((work + 255) / 256)), dim3(256), 0, s, a, rows);
    }
    return check_launch();
}

int mv_delta_chunked_ok(int n, int p) {
    return n > 0 && p > 0 && n <= 160 && p <= 256 && mv::delta_intra_lds(n) <= 158 * 1024;
}

int64_t mv_delta_scratch_floats(int n, int p) {
    const int64_t N = (n + 15) & ~15, P = (p + 15) & ~15;
    return 3 * mv::kDCh * N + mv::kDCh * P + mv::kDCh * mv::kDCh + N * P + N;
}

int mv_delta_rule(const float* qkv, int64_t ldq, const float* gate_in, int64_t lda, const float* z, int64_t ldz,
                  const float* beta, const float* dt_bias, const float* a_log, const float* norm, float* state,
                  void* out, int64_t ldo, const int32_t* row_start, const int32_t* row_len, const int32_t* row_ctx,
                  const int32_t* row_slot, int rows, int kv_heads, int heads, int n, int p, float eps, float* scratch,
                  const int32_t* ch_start, const int32_t* ch_len, const int32_t* row_ch0, const int32_t* row_nch,
                  int chunks, int max_len, int short_tokens, int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || kv_heads <= 0 || heads <= 0 || heads % kv_heads || n <= 0 || p <= 0 || chunks < 0)
        return MV_ERR_INVALID_ARG;
    if (p > 256 || n > kDeltaMaxN || rows > 65535 || chunks > 65535) return MV_ERR_UNSUPPORTED;
    if (rows == 0) return MV_OK;
    const int64_t cq = 2 * (int64_t)kv_heads * n + (int64_t)heads * p;
    if (!qkv || !gate_in || !z || !beta || !dt_bias || !a_log || !norm || !state || !out || !row_start || !row_len ||
        !row_ctx || !row_slot || ldq < cq || lda < (int64_t)heads * n || ldz < (int64_t)heads * p ||
        ldo < (int64_t)heads * p)
        return MV_ERR_INVALID_ARG;
    if (chunks > 0 && (!scratch || !ch_start || !ch_len || !row_ch0 || !row_nch || max_len <= 0 || !aligned16(scratch)))
        return MV_ERR_INVALID_ARG;
    if (chunks > 0 && !mv_delta_chunked_ok(n, p)) return MV_ERR_UNSUPPORTED;
    DeltaArgs a;
    a.qkv = qkv; a.a = gate_in; a.z = z; a.beta = beta; a.dt_bias = dt_bias; a.a_log = a_log; a.norm = norm;
    a.ldq = ldq; a.lda = lda; a.ldz = ldz; a.ldo = ldo; a.state = state; a.out = out;
    a.r = DeltaRows{nullptr, row_start, row_len, row_ctx, row_slot};
    a.K = kv_heads; a.H = heads; a.n = n; a.p = p; a.max_len = chunks > 0 ? max_len : 0; a.eps = eps;
    a.ch_start = ch_start; a.ch_len = ch_len; a.row_ch0 = row_ch0; a.row_nch = row_nch;
    a.vec = p % 16 == 0 && ldz % 4 == 0 && ldo % 4 == 0 && aligned16(z) && aligned16(out) && aligned16(norm);
    hipStream_t s = (hipStream_t)stream;
    if (chunks == 0 || short_tokens != 0) {
        int pw = 16;
        while (pw < p) pw *= 2;
        int nt = 256;
        while (nt < 1024 && (int64_t)n * pw > (int64_t)nt * 16) nt *= 2;
        const int ng = nt / pw, npt = (n + ng - 1) / ng;
        const size_t lds = ((size_t)3 * n + 2 * nt + ng + 8) * sizeof(float);
        const dim3 grid(heads, rows);
#define MV_DELTA_SCAN(M_)                                                                                       \
    do {                                                                                                       \
        if (f32) hipLaunchKernelGGL((delta_scan_kernel<true, M_>), grid, dim3(nt), lds, s, a, pw);               \
        else hipLaunchKernelGGL((delta_scan_kernel<false, M_>), grid, dim3(nt), lds, s, a, pw);                  \
    } while (0)
        if (npt <= 4) MV_DELTA_SCAN(4);
        else if (npt <= 8) MV_DELTA_SCAN(8);
        else if (npt <= 16) MV_DELTA_SCAN(16);
        else if (npt <= 32) MV_DELTA_SCAN(32);
        else if (npt <= 64) MV_DELTA_SCAN(64);
        else return MV_ERR_UNSUPPORTED;
#undef MV_DELTA_SCAN
    }
    if (chunks > 0) {
        const int64_t N = (n + 15) & ~15, P = (p + 15) & ~15, U = (int64_t)chunks * heads;
        a.qd = scratch;
        a.wk = a.qd + U * kDCh * N;
        a.kt = a.wk + U * kDCh * N;
        a.uv = a.kt + U * kDCh * N;
        a.bm = a.uv + U * kDCh * P;
        a.s0 = a.bm + U * kDCh * kDCh;
        a.gc = a.s0 + U * N * P;
        const size_t lds1 = delta_intra_lds(n), lds2 = (size_t)kDCh * (P + 4) * sizeof(float);
        static LdsOptIn o1, o2[2][6];
        if (int rc = ensure_dynamic_lds((const void*)delta_chunk_intra_kernel, lds1, o1)) return rc;
        hipLaunchKernelGGL(delta_chunk_intra_kernel, dim3(heads, chunks), dim3(kIntra), lds1, s, a);
        const dim3 gc(heads, (unsigned)(P / 16), rows);
        if (N == 128) hipLaunchKernelGGL((delta_chunk_carry_kernel<8, true>), gc, dim3(256), 0, s, a);
        else if (N == 64) hipLaunchKernelGGL((delta_chunk_carry_kernel<4, true>), gc, dim3(256), 0, s, a);
        else if (N <= 32) hipLaunchKernelGGL((delta_chunk_carry_kernel<2, false>), gc, dim3(256), 0, s, a);
        else if (N <= 64) hipLaunchKernelGGL((delta_chunk_carry_kernel<4, false>), gc, dim3(256), 0, s, a);
        else if (N <= 128) hipLaunchKernelGGL((delta_chunk_carry_kernel<8, false>), gc, dim3(256), 0, s, a);
        else hipLaunchKernelGGL((delta_chunk_carry_kernel<10, false>), gc, dim3(256), 0, s, a);
        const dim3 gi(heads, chunks);
#define MV_DELTA_INTER(F32_, PT_, FULL_, IDX_)                                                                             \
    do {                                                                                                               \
        const void* fn = (const void*)delta_chunk_inter_kernel<F32_, PT_, FULL_>;                                          \
        if (int rc = ensure_dynamic_lds(fn, lds2, o2[F32_][IDX_])) return rc;                                             \
        hipLaunchKernelGGL((delta_chunk_inter_kernel<F32_, PT_, FULL_>), gi, dim3(256), lds2, s, a);                       \
    } while (0)
#define MV_DELTA_INTER_P(F32_)                                                                                         \
    do {                                                                                                               \
        if (P == 128) MV_DELTA_INTER(F32_, 8, true, 0);                                                                  \
        else if (P == 64) MV_DELTA_INTER(F32_, 4, true, 1);                                                              \
        else if (P <= 32) MV_DELTA_INTER(F32_, 2, false, 2);                                                             \
        else if (P <= 64) MV_DELTA_INTER(F32_, 4, false, 3);                                                             \
        else if (P <= 128) MV_DELTA_INTER(F32_, 8, false, 4);                                                            \
        else MV_DELTA_INTER(F32_, 16, false, 5);                                                                         \
    } while (0)
        if (f32) MV_DELTA_INTER_P(true);
        else MV_DELTA_INTER_P(false);
#undef MV_DELTA_INTER_P
#undef MV_DELTA_INTER
    }
    return check_launch();
}

}  // extern "C"
