// Row-wise steps around an fp32 residual stream: layer stacks that keep the running sum of their
// sublayers in 32 bits and hand every projection a copy in the activation type (bf16, or fp32 when
// the whole model runs in 32 bits).
//
//   embed_scaled:        x = table[id] * scale                       (fp32), h = act(x), or act of a norm of x
//   postnorm_residual:   v = s1*y1 (+ s2*y2); x += v / sqrt(mean(v^2) + eps) * (1 + w); h = act(x)
//                        (the norm sits on the SUBLAYER'S OUTPUT, its weight is stored as an offset
//                        from one); optionally a bias inside v, a factor on what is added, and h = act of the NEXT
//                        sublayer's norm of the new x
//   offset_rmsnorm_gather: out = act( x[idx] / sqrt(mean(x[idx]^2) + eps) * (1 + w) )
//   relu_squared:        out = act( max(v, 0)^2 )
//   softcap:             v = cap * tanh(v / cap)
//   dyt_shift:           n = tanh(alpha x) w + b (a norm without statistics); h_t = act( n_t + (n_(t-1) - n_t) mix ),
//                        the last n of every row kept per state slot for the row's next step
//   dyt_gather:          out = act( tanh(alpha x[idx]) w + b )
//   dyt_residual:        x += tanh(alpha y) w + b; h = act(x), or act of the next sublayer's norm of x
//   unitnorm_residual:   x += y / sqrt(mean(y^2) + eps) * w; h = act(x)     (plain weight)
//   rmsnorm_rows:        out = act( v / sqrt(mean(v^2) + eps) * w )         (plain weight, rows of any stride)
//   gelu_gate_rows:      out = act( gelu_tanh(a) * table[id][off .. off+n) )
//   silu_mul:            out = act( silu(a[:, :n]) * a[:, n:2n] )
//   sigmoid_gate:        out = act( a * sigmoid(g) )   (g == NULL: act(a))
//   embed_pair:          x = table[id] * scale + pairs[(prev * mul_prev + id * mul_cur) mod buckets]   (a hashed
//                        table over pairs of neighbouring tokens; row `buckets` where a token has no predecessor);
//                        optionally h = act( x / sqrt(mean(x^2) + eps) * w ), the first layer's norm
//   add_rmsnorm:         x += y1 (+ y2); h = act( x / sqrt(mean(x^2) + eps) * w )   (the sublayers of a parallel
//                        layer enter the stream together and the next layer's norm comes out of the same launch)
//   rmsnorm_gather:      out = act( x[idx] / sqrt(mean(x[idx]^2) + eps) * (offset + w) )
//   gated_act:           out = act( f(a[:, :n]) * a[:, n:2n] ), f = SiLU or the tanh form of GELU; or the clamped
//                        gate  g' = min(g, limit), u' = clamp(u, +-limit): out = act( g' sigmoid(slope g') (u' + 1) )
//   gated_residual_norm: the residual step of a pre-norm layer whose sublayer outputs pass a sigmoid gate:
//                        x += y * sigmoid(g + b)  (mode 1), or  x = y + b  (mode 2: a new pass of a looped span
//                        starts from a projection plus a per-pass vector); then n = x / sqrt(mean(x^2) + eps) *
//                        (offset + w) as fp32 (what a convolution over time reads) and / or in the activation type
//   cast_concat:         out = act( [a | b] )   (two fp32 streams side by side as one projection's operand)
//   gelu_tanh:           out = act( gelu(in) ), the tanh form
//   scale:               v *= s
//   layernorm_residual:  x += LN(v) with LN(v) = (v - mean) / sqrt(mean((v - mean)^2) + eps) * w, h = act(x) or, with w2,
//                        act of a second layer norm of the new x.  v is one sublayer's output; or s times the sum of two
//                        branches, each first divided by its root mean square and weighted; or the weighted sum of a
//                        token's routed expert rows (+ a shared expert's row)
//   layernorm_gather:    out = act( LN(x[idx]) )
// All arithmetic is fp32 with the library's exact division, square root and tanh.
#include "common.h"

namespace mv {

template <bool F32> struct Act;
template <> struct Act<true> {
    typedef float T;
    static __device__ __forceinline__ float ld(const float* p) { return *p; }
    static __device__ __forceinline__ void st(float* p, float v) { *p = v; }
};
template <> struct Act<false> {
    typedef uint16_t T;
    static __device__ __forceinline__ float ld(const uint16_t* p) { return bf16_bits_to_f32(*p); }
    static __device__ __forceinline__ void st(uint16_t* p, float v) { *p = (uint16_t)f32_to_bf16_bits(v); }
};

// w != NULL: h receives x / sqrt(mean(x^2) + eps) * (offset + w), the first layer's norm, instead of x itself
template <bool F32>
__global__ __launch_bounds__(1024) void embed_scaled_kernel(const void* table_, const int* ids, float* x, int64_t ldx,
                                                           void* h_, int64_t ldh, int n, int vocab, float scale,
                                                           const float* w, float eps, float offset) {
    typedef typename Act<F32>::T T;
    __shared__ float red[16];
    const T* table = (const T*)table_;
    T* h = (T*)h_;
    const int row = blockIdx.x;
    int id = ids[row];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
    float ss = 0.f;
    for (int c = threadIdx.x; c < n; c += blockDim.x) {
        const float v = Act<F32>::ld(table + (int64_t)id * n + c) * scale;
        x[(int64_t)row * ldx + c] = v;
        if (!w) Act<F32>::st(h + (int64_t)row * ldh + c, v);
        ss += v * v;
    }
    if (!w) return;
    ss = block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)n + eps);
    for (int c = threadIdx.x; c < n; c += blockDim.x) {
        const float v = Act<F32>::ld(table + (int64_t)id * n + c) * scale;
        Act<F32>::st(h + (int64_t)row * ldh + c, (v * inv) * (offset + w[c]));
    }
}

struct PostnormArgs {
    const float *y1, *y2, *bias, *w, *w2;
    int64_t ld1, ld2, ldx, ldh;
    float s1, s2, eps, mult;
    float* x;
    void* h;
    int n;
};

template <bool F32>
__global__ __launch_bounds__(256) void postnorm_residual_kernel(PostnormArgs a) {
    typedef typename Act<F32>::T T;
    __shared__ float red[4];
    T* h = (T*)a.h;
    const int row = blockIdx.x;
    const float* y1 = a.y1 + (int64_t)row * a.ld1;
    const float* y2 = a.y2 ? a.y2 + (int64_t)row * a.ld2 : nullptr;
    auto value = [&](int c) {
        float v = y2 ? a.s1 * y1[c] + a.s2 * y2[c] : a.s1 * y1[c];
        return a.bias ? v + a.bias[c] : v;
    };
    float ss = 0.f;
    for (int c = threadIdx.x; c < a.n; c += 256) {
        const float v = value(c);
        ss += v * v;
    }
    ss = block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)a.n + a.eps);
    float* xr = a.x + (int64_t)row * a.ldx;
    float s2 = 0.f;
    for (int c = threadIdx.x; c < a.n; c += 256) {
        const float s = xr[c] + a.mult * ((value(c) * inv) * (1.0f + a.w[c]));
        xr[c] = s;
        if (!a.w2) Act<F32>::st(h + (int64_t)row * a.ldh + c, s);
        s2 += s * s;
    }
    if (!a.w2) return;
    s2 = block_sum(s2, red);
    const float inv2 = 1.0f / sqrtf(s2 / (float)a.n + a.eps);
    for (int c = threadIdx.x; c < a.n; c += 256)
        Act<F32>::st(h + (int64_t)row * a.ldh + c, (xr[c] * inv2) * (1.0f + a.w2[c]));
}

// the same with the row in registers: n a multiple of 4 up to 4 * threads * NV, every row 16-byte aligned
template <bool F32, int NV>
__global__ __launch_bounds__(1024) void postnorm_residual_reg_kernel(PostnormArgs a) {
    __shared__ float red[16];
    const int row = blockIdx.x, tid = threadIdx.x, n4 = a.n / 4;
    const float4* y1 = reinterpret_cast<const float4*>(a.y1 + (int64_t)row * a.ld1);
    const float4* y2 = a.y2 ? reinterpret_cast<const float4*>(a.y2 + (int64_t)row * a.ld2) : nullptr;
    const float4* bias = reinterpret_cast<const float4*>(a.bias);
    const float4* w = reinterpret_cast<const float4*>(a.w);
    const float4* w2 = reinterpret_cast<const float4*>(a.w2);
    float4* xr = reinterpret_cast<float4*>(a.x + (int64_t)row * a.ldx);
    float4 v[NV], xv[NV];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = tid + (int)blockDim.x * i;
        v[i] = xv[i] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (c < n4) {
            const float4 p = y1[c];
            v[i] = make_float4(a.s1 * p.x, a.s1 * p.y, a.s1 * p.z, a.s1 * p.w);
            if (y2) {
                const float4 q = y2[c];
                v[i].x += a.s2 * q.x; v[i].y += a.s2 * q.y; v[i].z += a.s2 * q.z; v[i].w += a.s2 * q.w;
            }
            if (bias) {
                const float4 q = bias[c];
                v[i].x += q.x; v[i].y += q.y; v[i].z += q.z; v[i].w += q.w;
            }
            xv[i] = xr[c];
        }
        ss += v[i].x * v[i].x + v[i].y * v[i].y + v[i].z * v[i].z + v[i].w * v[i].w;
    }
    ss = block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)a.n + a.eps);
    float s2 = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = tid + (int)blockDim.x * i;
        if (c < n4) {
            const float4 q = w[c];
            xv[i].x += a.mult * ((v[i].x * inv) * (1.0f + q.x));
            xv[i].y += a.mult * ((v[i].y * inv) * (1.0f + q.y));
            xv[i].z += a.mult * ((v[i].z * inv) * (1.0f + q.z));
            xv[i].w += a.mult * ((v[i].w * inv) * (1.0f + q.w));
            xr[c] = xv[i];
        }
        s2 += xv[i].x * xv[i].x + xv[i].y * xv[i].y + xv[i].z * xv[i].z + xv[i].w * xv[i].w;
    }
    float inv2 = 1.0f;
    if (a.w2) {
        s2 = block_sum(s2, red);
        inv2 = 1.0f / sqrtf(s2 / (float)a.n + a.eps);
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = tid + (int)blockDim.x * i;
        if (c >= n4) continue;
        float4 o = xv[i];
        if (a.w2) {
            const float4 q = w2[c];
            o.x = (o.x * inv2) * (1.0f + q.x);
            o.y = (o.y * inv2) * (1.0f + q.y);
            o.z = (o.z * inv2) * (1.0f + q.z);
            o.w = (o.w * inv2) * (1.0f + q.w);
        }
        if (F32) {
            reinterpret_cast<float4*>((float*)a.h + (int64_t)row * a.ldh)[c] = o;
        } else {
            uint2 pk;
            pk.x = pack_bf16x2(o.x, o.y);
            pk.y = pack_bf16x2(o.z, o.w);
            reinterpret_cast<uint2*>((uint16_t*)a.h + (int64_t)row * a.ldh)[c] = pk;
        }
    }
}

template <bool F32>
__global__ __launch_bounds__(256) void offset_rmsnorm_gather_kernel(const float* x, int64_t ldx, const int* idx,
                                                                    const float* w, float eps, float offset,
                                                                    void* out_, int64_t ldo, int n) {
    typedef typename Act<F32>::T T;
    __shared__ float red[4];
    T* out = (T*)out_;
    const int row = blockIdx.x;
    const float* a = x + (int64_t)(idx ? idx[row] : row) * ldx;
    float ss = 0.f;
    for (int c = threadIdx.x; c < n; c += 256) ss += a[c] * a[c];
    ss = block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)n + eps);
    for (int c = threadIdx.x; c < n; c += 256) Act<F32>::st(out + (int64_t)row * ldo + c, (a[c] * inv) * (offset + w[c]));
}

template <bool F32>
__global__ __launch_bounds__(256) void relu_squared_kernel(const float* in, int64_t ldi, void* out_, int64_t ldo,
                                                           int n) {
    typedef typename Act<F32>::T T;
    T* out = (T*)out_;
    const int row = blockIdx.x;
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c >= n) return;
    const float v = fmaxf(in[(int64_t)row * ldi + c], 0.f);
    Act<F32>::st(out + (int64_t)row * ldo + c, v * v);
}

// the same, four values a thread (n a multiple of 4, rows aligned)
template <bool F32>
__global__ __launch_bounds__(256) void relu_squared4_kernel(const float* in, int64_t ldi, void* out_, int64_t ldo, int n4) {
    const int row = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
    if (c >= n4) return;
    float4 v = reinterpret_cast<const float4*>(in + (int64_t)row * ldi)[c];
    v = make_float4(fmaxf(v.x, 0.f), fmaxf(v.y, 0.f), fmaxf(v.z, 0.f), fmaxf(v.w, 0.f));
    v = make_float4(v.x * v.x, v.y * v.y, v.z * v.z, v.w * v.w);
    if (F32) reinterpret_cast<float4*>((float*)out_ + (int64_t)row * ldo)[c] = v;
    else reinterpret_cast<uint2*>((uint16_t*)out_ + (int64_t)row * ldo)[c] = make_uint2(pack_bf16x2(v.x, v.y), pack_bf16x2(v.z, v.w));
}

__global__ __launch_bounds__(256) void softcap_kernel(float* v, int64_t count, float cap) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i < count) v[i] = cap * tanhf(v[i] / cap);
}

// ---- Dynamic Tanh norm, token shift ------------------------------------------------------------------
// One workgroup per token.  n_(t-1) of a row's first token is the slot's kept vector (zeros when the
// sequence holds nothing yet); the workgroup of that first token also writes the row's LAST n into the
// slot, so that nobody else touches the slot in this launch.
template <bool F32>
__global__ __launch_bounds__(256) void dyt_shift_kernel(const float* x, int64_t ldx, const float* w, const float* b,
                                                        const float* alpha, const float* mix, float* state,
                                                        void* h_, int64_t ldh, const int* tok_row,
                                                        const int* row_start, const int* row_len, const int* row_ctx,
                                                        const int* row_slot, int n) {
    typedef typename Act<F32>::T T;
    T* h = (T*)h_;
    const int t = blockIdx.x, r = tok_row[t];
    const int first = row_start[r], len = row_len[r];
    const float al = alpha[0];
    const float* cur = x + (int64_t)t * ldx;
    const bool head = t == first;
    float* kept = state + (int64_t)row_slot[r] * n;
    const bool carried = row_ctx[r] > 0;
    const float* prev = x + (int64_t)(t - 1) * ldx;
    const float* last = x + (int64_t)(first + len - 1) * ldx;
    // one value per thread (blockIdx.y walks the row): a row alone in its step is spread over many workgroups
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c < n) {
        const float nc = fmaf(tanhf(al * cur[c]), w[c], b[c]);
        float np;
        if (head) np = carried ? kept[c] : 0.f;
        else np = fmaf(tanhf(al * prev[c]), w[c], b[c]);
        Act<F32>::st(h + (int64_t)t * ldh + c, fmaf(np - nc, mix[c], nc));
        if (head) kept[c] = len == 1 ? nc : fmaf(tanhf(al * last[c]), w[c], b[c]);
    }
}

template <bool F32>
__global__ __launch_bounds__(256) void dyt_gather_kernel(const float* x, int64_t ldx, const int* idx, const float* w,
                                                         const float* b, const float* alpha, void* out_, int64_t ldo,
                                                         int n) {
    typedef typename Act<F32>::T T;
    T* out = (T*)out_;
    const int row = blockIdx.x;
    const float* a = x + (int64_t)(idx ? idx[row] : row) * ldx;
    const float al = alpha[0];
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c < n) Act<F32>::st(out + (int64_t)row * ldo + c, fmaf(tanhf(al * a[c]), w[c], b[c]));
}

// w2 != NULL: h receives the NEXT sublayer's norm of the new x, tanh(alpha2 x) w2 + b2, instead of x itself
template <bool F32>
__global__ __launch_bounds__(256) void dyt_residual_kernel(const float* y, int64_t ldy, const float* w, const float* b,
                                                           const float* alpha, float* x, int64_t ldx, void* h_,
                                                           int64_t ldh, int n, const float* w2, const float* b2,
                                                           const float* alpha2) {
    typedef typename Act<F32>::T T;
    T* h = (T*)h_;
    const int row = blockIdx.x;
    const float al = alpha[0];
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c < n) {
        const float s = x[(int64_t)row * ldx + c] + fmaf(tanhf(al * y[(int64_t)row * ldy + c]), w[c], b[c]);
        x[(int64_t)row * ldx + c] = s;
        if (h) Act<F32>::st(h + (int64_t)row * ldh + c, w2 ? fmaf(tanhf(alpha2[0] * s), w2[c], b2[c]) : s);
    }
}

template <bool F32>
__global__ __launch_bounds__(256) void unitnorm_residual_kernel(const float* y, int64_t ldy, const float* w, float eps,
                                                                float* x, int64_t ldx, void* h_, int64_t ldh, int n) {
    typedef typename Act<F32>::T T;
    __shared__ float red[4];
    T* h = (T*)h_;
    const int row = blockIdx.x;
    const float* a = y + (int64_t)row * ldy;
    float ss = 0.f;
#pragma unroll 4
    for (int c = threadIdx.x; c < n; c += 256) ss += a[c] * a[c];
    ss = block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)n + eps);
#pragma unroll 4
    for (int c = threadIdx.x; c < n; c += 256) {
        const float s = x[(int64_t)row * ldx + c] + (a[c] * inv) * w[c];
        x[(int64_t)row * ldx + c] = s;
        if (h) Act<F32>::st(h + (int64_t)row * ldh + c, s);
    }
}

// one wave per row of `n` values (rows may be heads of a wider buffer: row r starts at (r / per) * ld + (r % per) * n)
template <bool F32>
__global__ __launch_bounds__(256) void rmsnorm_rows_kernel(const float* v, int64_t ld, int per, const float* w,
                                                           float eps, void* out_, int64_t ldo, int64_t rows, int n) {
    typedef typename Act<F32>::T T;
    T* out = (T*)out_;
    const int64_t r = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    const int lane = threadIdx.x & 63;
    if (r >= rows) return;
    const float* a = v + (r / per) * ld + (r % per) * n;
    T* o = out + (r / per) * ldo + (r % per) * n;
    float ss = 0.f;
#pragma unroll 4
    for (int c = lane; c < n; c += 64) ss += a[c] * a[c];
    ss = wave_sum(ss);
    const float inv = 1.0f / sqrtf(ss / (float)n + eps);
#pragma unroll 4
    for (int c = lane; c < n; c += 64) Act<F32>::st(o + c, (a[c] * inv) * w[c]);
}

template <bool F32>
__global__ __launch_bounds__(256) void gelu_gate_rows_kernel(const float* a, int64_t lda, const void* table_,
                                                             int64_t ldt, int off, const int* ids, int vocab,
                                                             void* out_, int64_t ldo, int n) {
    typedef typename Act<F32>::T T;
    const T* table = (const T*)table_;
    T* out = (T*)out_;
    const int row = blockIdx.x;
    int id = ids[row];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c < n) {
        const float e = Act<F32>::ld(table + (int64_t)id * ldt + off + c);
        Act<F32>::st(out + (int64_t)row * ldo + c, gelu_tanh_f(a[(int64_t)row * lda + c]) * e);
    }
}

template <bool F32>
__global__ __launch_bounds__(256) void silu_mul_kernel(const float* a, int64_t lda, void* out_, int64_t ldo, int n) {
    typedef typename Act<F32>::T T;
    T* out = (T*)out_;
    const int64_t row = blockIdx.x;
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c >= n) return;
    const float g = a[row * lda + c], u = a[row * lda + n + c];
    Act<F32>::st(out + row * ldo + c, (g / (1.0f + expf(-g))) * u);
}

template <bool F32>
__global__ __launch_bounds__(256) void sigmoid_gate_kernel(const float* a, int64_t lda, const float* g, int64_t ldg,
                                                           void* out_, int64_t ldo, int n) {
    typedef typename Act<F32>::T T;
    T* out = (T*)out_;
    const int64_t row = blockIdx.x;
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c >= n) return;
    float v = a[row * lda + c];
    if (g) v = v / (1.0f + expf(-g[row * ldg + c]));
    Act<F32>::st(out + row * ldo + c, v);
}

// ---- pair-hashed embedding, parallel layers behind one norm, gated activations ----------------------------
template <bool F32>
__global__ __launch_bounds__(256) void embed_pair_kernel(const void* table_, const void* pairs_, const int* ids,
                                                         const int* prev, float* x, int64_t ldx, int n, int vocab,
                                                         int64_t buckets, int64_t mul_prev, int64_t mul_cur,
                                                         float scale, const float* norm_w, float eps, void* h_,
                                                         int64_t ldh) {
    typedef typename Act<F32>::T T;
    __shared__ float red[4];
    const T* table = (const T*)table_;
    const T* pairs = (const T*)pairs_;
    const int row = blockIdx.x;
    int id = ids[row];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
    const int pv = prev[row];
    // every factor reduced first: the products stay below 2^62 for any 31-bit bucket count
    const int64_t r = pv < 0 ? buckets
                             : (((int64_t)pv % buckets) * (mul_prev % buckets) % buckets +
                                ((int64_t)id % buckets) * (mul_cur % buckets) % buckets) % buckets;
    float ss = 0.f;
    for (int c = threadIdx.x; c < n; c += 256) {
        const float v = Act<F32>::ld(table + (int64_t)id * n + c) * scale + Act<F32>::ld(pairs + r * n + c);
        x[(int64_t)row * ldx + c] = v;
        ss += v * v;
    }
    if (!norm_w) return;
    // the first layer's norm of the row out of the same launch
    ss = block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)n + eps);
    for (int c = threadIdx.x; c < n; c += 256)
        Act<F32>::st((T*)h_ + (int64_t)row * ldh + c, (x[(int64_t)row * ldx + c] * inv) * norm_w[c]);
}

template <bool F32>
__global__ __launch_bounds__(256) void add_rmsnorm_kernel(const float* y1, int64_t ld1, const float* y2, int64_t ld2,
                                                          float* x, int64_t ldx, const float* w, float eps, void* h_,
                                                          int64_t ldh, int n) {
    typedef typename Act<F32>::T T;
    __shared__ float red[4];
    T* h = (T*)h_;
    const int row = blockIdx.x;
    float* xr = x + (int64_t)row * ldx;
    float ss = 0.f;
#pragma unroll 4
    for (int c = threadIdx.x; c < n; c += 256) {
        float v = xr[c];
        if (y1) {
            v += y2 ? y1[(int64_t)row * ld1 + c] + y2[(int64_t)row * ld2 + c] : y1[(int64_t)row * ld1 + c];
            xr[c] = v;
        }
        ss += v * v;
    }
    if (!w) return;
    ss = block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)n + eps);
#pragma unroll 4
    for (int c = threadIdx.x; c < n; c += 256) Act<F32>::st(h + (int64_t)row * ldh + c, (xr[c] * inv) * w[c]);
}

template <bool F32>
__global__ __launch_bounds__(256) void gated_act_kernel(const float* a, int64_t lda, void* out_, int64_t ldo, int n,
                                                        int kind, float limit, float slope) {
    typedef typename Act<F32>::T T;
    T* out = (T*)out_;
    const int64_t row = blockIdx.x;
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c >= n) return;
    Act<F32>::st(out + row * ldo + c, gated_act_f(a[row * lda + c], a[row * lda + n + c], kind, limit, slope));
}

// four values a thread: n a multiple of 4, rows 16-byte aligned
template <bool F32>
__global__ __launch_bounds__(256) void gated_act4_kernel(const float* a, int64_t lda, void* out, int64_t ldo, int n,
                                                         int kind, float limit, float slope) {
    const int64_t row = blockIdx.x;
    const int c = (blockIdx.y * 256 + threadIdx.x) * 4;
    if (c >= n) return;
    const float4 g = *reinterpret_cast<const float4*>(a + row * lda + c);
    const float4 u = *reinterpret_cast<const float4*>(a + row * lda + n + c);
    const float4 o = make_float4(gated_act_f(g.x, u.x, kind, limit, slope), gated_act_f(g.y, u.y, kind, limit, slope),
                                 gated_act_f(g.z, u.z, kind, limit, slope), gated_act_f(g.w, u.w, kind, limit, slope));
    if (F32) *reinterpret_cast<float4*>((float*)out + row * ldo + c) = o;
    else *reinterpret_cast<uint2*>((uint16_t*)out + row * ldo + c) = make_uint2(pack_bf16x2(o.x, o.y), pack_bf16x2(o.z, o.w));
}


// mode 0: x as it is; 1: x += y * sigmoid(g + b); 2: x = y + b.  w != NULL: the norm of the new x, to n32 (fp32)
// and / or h (activation type)
template <bool F32>
__global__ __launch_bounds__(256) void gated_residual_norm_kernel(const float* y, int64_t ldy, const float* g,
                                                                  int64_t ldg, const float* b, int mode, float* x,
                                                                  int64_t ldx, const float* w, float eps, float offset,
                                                                  float* n32, int64_t ldn, void* h_, int64_t ldh,
                                                                  int n) {
    typedef typename Act<F32>::T T;
    __shared__ float red[4];
    T* h = (T*)h_;
    const int64_t row = blockIdx.x;
    float* xr = x + row * ldx;
    float ss = 0.f;
#pragma unroll 4
    for (int c = threadIdx.x; c < n; c += 256) {
        float v;
        if (mode == 1) {
            const float z = g[row * ldg + c] + (b ? b[c] : 0.f);
            v = fmaf(y[row * ldy + c], 1.0f / (1.0f + expf(-z)), xr[c]);
            xr[c] = v;
        } else if (mode == 2) {
            v = y[row * ldy + c] + (b ? b[c] : 0.f);
            xr[c] = v;
        } else {
            v = xr[c];
        }
        ss += v * v;
    }
    if (!w) return;
    ss = block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)n + eps);
#pragma unroll 4
    for (int c = threadIdx.x; c < n; c += 256) {
        const float v = (xr[c] * inv) * (offset + w[c]);
        if (n32) n32[row * ldn + c] = v;
        if (h) Act<F32>::st(h + row * ldh + c, v);
    }
}

template <bool F32>
__global__ __launch_bounds__(256) void cast_concat_kernel(const float* a, int64_t lda, const float* b, int64_t ldb,
                                                          void* out_, int64_t ldo, int n) {
    typedef typename Act<F32>::T T;
    T* out = (T*)out_;
    const int64_t row = blockIdx.x;
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c >= 2 * n) return;
    Act<F32>::st(out + row * ldo + c, c < n ? a[row * lda + c] : b[row * ldb + (c - n)]);
}

template <bool F32>
__global__ __launch_bounds__(256) void gelu_tanh_kernel(const float* in, int64_t ldi, void* out_, int64_t ldo, int n) {
    typedef typename Act<F32>::T T;
    T* out = (T*)out_;
    const int64_t row = blockIdx.x;
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c < n) Act<F32>::st(out + row * ldo + c, gelu_tanh_f(in[row * ldi + c]));
}

__global__ __launch_bounds__(256) void scale_kernel(float* v, int64_t count, float s) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i < count) v[i] *= s;
}

// ---- layer norm on a sublayer's output ----------------------------------------------------------------
struct LayernormArgs {
    const float *y1, *r1, *y2, *r2;      // r1 / r2: weights of the two branches' RMS norms (y2 == NULL: y1 as it is)
    const int* place;                    // experts: rows of y1 the token's choices lie in, [rows, top]
    const float* wts;                    // [rows, top]
    const float *w, *w2;
    int64_t ld1, ld2, ldx, ldh;
    float s, eps;
    float* x;
    void* h;
    int n, top;
};

// The row in registers, VEC (4: every row 16-byte aligned, n a multiple of 4; or 1) values a thread and turn, NV turns.
template <bool F32, int VEC, int NV>
__global__ __launch_bounds__(1024) void layernorm_residual_kernel(LayernormArgs a) {
    typedef typename Act<F32>::T T;
    __shared__ float red[16], red2[16];
    const int row = blockIdx.x, tid = threadIdx.x, NT = blockDim.x, cnt = a.n / VEC;
    auto load = [&](const float* p, int c, float (&o)[VEC]) {
        if (VEC == 4) {
            const float4 q = reinterpret_cast<const float4*>(p)[c];
            o[0] = q.x; o[VEC > 1 ? 1 : 0] = q.y; o[VEC > 2 ? 2 : 0] = q.z; o[VEC > 3 ? 3 : 0] = q.w;
        } else {
            o[0] = p[c];
        }
    };
    float v[NV][VEC], xv[NV][VEC];
    float* xr = a.x + (int64_t)row * a.ldx;
    const float* y1 = a.y1 + (int64_t)row * a.ld1;
    const float* y2 = a.y2 ? a.y2 + (int64_t)row * a.ld2 : nullptr;
    const bool branches = y2 && !a.place;
    float u[NV][VEC];                    // the second branch
    float s1 = 0.f, s2 = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = tid + NT * i;
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[i][j] = u[i][j] = xv[i][j] = 0.f;
        if (c >= cnt) continue;
        load(xr, c, xv[i]);
        if (a.place) {
            if (y2) load(y2, c, v[i]);
        } else {
            load(y1, c, v[i]);
            if (y2) load(y2, c, u[i]);
        }
    }
    if (a.place) {
        constexpr int kB = 4;            // expert rows in flight together
        for (int k0 = 0; k0 < a.top; k0 += kB) {
            const float* e[kB];
            float ew[kB];
#pragma unroll
            for (int k = 0; k < kB; ++k) {
                const int64_t at = (int64_t)row * a.top + (k0 + k < a.top ? k0 + k : k0);
                e[k] = a.y1 + (int64_t)a.place[at] * a.ld1;
                ew[k] = k0 + k < a.top ? a.wts[at] : 0.f;
            }
#pragma unroll
            for (int i = 0; i < NV; ++i) {
                const int c = tid + NT * i;
                if (c >= cnt) continue;
                float q[kB][VEC];
#pragma unroll
                for (int k = 0; k < kB; ++k) load(e[k], c, q[k]);
#pragma unroll
                for (int k = 0; k < kB; ++k)
#pragma unroll
                    for (int j = 0; j < VEC; ++j) v[i][j] = fmaf(ew[k], q[k][j], v[i][j]);
            }
        }
    }
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
            s1 += branches ? v[i][j] * v[i][j] : v[i][j];
            s2 += u[i][j] * u[i][j];
        }
    if (branches) {
        s1 = wave_sum(s1);
        s2 = wave_sum(s2);
        if ((tid & 63) == 0) {
            red[tid >> 6] = s1;
            red2[tid >> 6] = s2;
        }
        __syncthreads();
        s1 = s2 = 0.f;
        for (int i = 0; i < NT / 64; ++i) {
            s1 += red[i];
            s2 += red2[i];
        }
        __syncthreads();
        const float i1 = 1.0f / sqrtf(s1 / (float)a.n + a.eps), i2 = 1.0f / sqrtf(s2 / (float)a.n + a.eps);
        s1 = 0.f;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = tid + NT * i;
            if (c >= cnt) continue;
            float w1[VEC], w2[VEC];
            load(a.r1, c, w1);
            load(a.r2, c, w2);
#pragma unroll
            for (int j = 0; j < VEC; ++j) {
                v[i][j] = a.s * ((v[i][j] * i1) * w1[j] + (u[i][j] * i2) * w2[j]);
                s1 += v[i][j];
            }
        }
    }
    // mean, then the squared deviations from it; the row stays in registers
    const float mean = block_sum(s1, red) / (float)a.n;
    float sq = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
            v[i][j] = tid + NT * i < cnt ? v[i][j] - mean : 0.f;
            sq += v[i][j] * v[i][j];
        }
    const float inv = 1.0f / sqrtf(block_sum(sq, red) / (float)a.n + a.eps);
    float sx = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = tid + NT * i;
        if (c >= cnt) continue;
        float w[VEC];
        load(a.w, c, w);
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
            xv[i][j] += (v[i][j] * inv) * w[j];
            sx += xv[i][j];
        }
        if (VEC == 4) reinterpret_cast<float4*>(xr)[c] = make_float4(xv[i][0], xv[i][VEC > 1 ? 1 : 0], xv[i][VEC > 2 ? 2 : 0], xv[i][VEC > 3 ? 3 : 0]);
        else xr[c] = xv[i][0];
    }
    float inv2 = 1.f, mean2 = 0.f;
    if (a.w2) {
        mean2 = block_sum(sx, red) / (float)a.n;
        sq = 0.f;
#pragma unroll
        for (int i = 0; i < NV; ++i)
#pragma unroll
            for (int j = 0; j < VEC; ++j) {
                const float d = tid + NT * i < cnt ? xv[i][j] - mean2 : 0.f;
                sq += d * d;
            }
        inv2 = 1.0f / sqrtf(block_sum(sq, red) / (float)a.n + a.eps);
    }
    if (!a.h) return;
    T* h = (T*)a.h + (int64_t)row * a.ldh;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = tid + NT * i;
        if (c >= cnt) continue;
        float o[VEC];
        if (a.w2) {
            load(a.w2, c, o);
#pragma unroll
            for (int j = 0; j < VEC; ++j) o[j] = ((xv[i][j] - mean2) * inv2) * o[j];
        } else {
#pragma unroll
            for (int j = 0; j < VEC; ++j) o[j] = xv[i][j];
        }
        if (VEC == 4) {
            const float o1 = o[VEC > 1 ? 1 : 0], o2 = o[VEC > 2 ? 2 : 0], o3 = o[VEC > 3 ? 3 : 0];
            if (F32) reinterpret_cast<float4*>(h)[c] = make_float4(o[0], o1, o2, o3);
            else reinterpret_cast<uint2*>(h)[c] = make_uint2(pack_bf16x2(o[0], o1), pack_bf16x2(o2, o3));
        } else {
            Act<F32>::st(h + c, o[0]);
        }
    }
}

template <bool F32>
__global__ __launch_bounds__(256) void layernorm_gather_kernel(const float* x, int64_t ldx, const int* idx, const float* w,
                                                               float eps, void* out_, int64_t ldo, int n) {
    typedef typename Act<F32>::T T;
    __shared__ float red[4];
    T* out = (T*)out_;
    const int row = blockIdx.x;
    const float* a = x + (int64_t)(idx ? idx[row] : row) * ldx;
    float s = 0.f;
    for (int c = threadIdx.x; c < n; c += 256) s += a[c];
    const float mean = block_sum(s, red) / (float)n;
    s = 0.f;
    for (int c = threadIdx.x; c < n; c += 256) s += (a[c] - mean) * (a[c] - mean);
    const float inv = 1.0f / sqrtf(block_sum(s, red) / (float)n + eps);
    for (int c = threadIdx.x; c < n; c += 256) Act<F32>::st(out + (int64_t)row * ldo + c, ((a[c] - mean) * inv) * w[c]);
}

}  // namespace mv

extern "C" {

int mv_embed_scaled(const void* table, const int32_t* ids, float* x, int64_t ldx, void* h, int64_t ldh, int rows,
                    int n, int vocab, float scale, const float* norm_w, float eps, float offset, int f32,
                    mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0 || vocab <= 0) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!table || !ids || !x || !h || ldx < n || ldh < n) return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    const int nt = rows <= 512 && n > 1024 ? 1024 : 256;
    if (f32) hipLaunchKernelGGL(embed_scaled_kernel<true>, dim3(rows), dim3(nt), 0, s, table, ids, x, ldx, h, ldh, n, vocab, scale, norm_w, eps, offset);
    else hipLaunchKernelGGL(embed_scaled_kernel<false>, dim3(rows), dim3(nt), 0, s, table, ids, x, ldx, h, ldh, n, vocab, scale, norm_w, eps, offset);
    return check_launch();
}

int mv_postnorm_residual(const float* y1, int64_t ld1, const float* y2, int64_t ld2, float s1, float s2,
                         const float* bias, const float* w, float eps, float mult, const float* next_w, float* x,
                         int64_t ldx, void* h, int64_t ldh, int rows, int n, int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!y1 || !w || !x || !h || ld1 < n || (y2 && ld2 < n) || ldx < n || ldh < n) return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    PostnormArgs a;
    a.y1 = y1; a.y2 = y2; a.bias = bias; a.w = w; a.w2 = next_w;
    a.ld1 = ld1; a.ld2 = ld2; a.ldx = ldx; a.ldh = ldh;
    a.s1 = s1; a.s2 = s2; a.eps = eps; a.mult = mult;
    a.x = x; a.h = h; a.n = n;
    const bool even = n % 4 == 0 && ld1 % 4 == 0 && ldx % 4 == 0 && ldh % 4 == 0 && (!y2 || ld2 % 4 == 0) && aligned16(y1) &&
                      aligned16(x) && aligned16(h) && aligned16(w) && (!y2 || aligned16(y2)) &&
                      (!bias || aligned16(bias)) && (!next_w || aligned16(next_w));
    // a row of a short step has its workgroup to itself on a compute unit: more threads, fewer values each
    const int nt = rows > 512 || n <= 1024 ? 256 : n <= 2048 ? 512 : 1024;
#define MV_POSTNORM(NV_)                                                                                              \
    do {                                                                                                              \
        if (f32) hipLaunchKernelGGL((postnorm_residual_reg_kernel<true, NV_>), dim3(rows), dim3(nt), 0, s, a);         \
        else hipLaunchKernelGGL((postnorm_residual_reg_kernel<false, NV_>), dim3(rows), dim3(nt), 0, s, a);            \
    } while (0)
    if (even && n <= 4 * nt) MV_POSTNORM(1);
    else if (even && n <= 8 * nt) MV_POSTNORM(2);
    else if (even && n <= 16 * nt) MV_POSTNORM(4);
    else if (even && n <= 32 * nt) MV_POSTNORM(8);
    else if (f32) hipLaunchKernelGGL(postnorm_residual_kernel<true>, dim3(rows), dim3(256), 0, s, a);
    else hipLaunchKernelGGL(postnorm_residual_kernel<false>, dim3(rows), dim3(256), 0, s, a);
#undef MV_POSTNORM
    return check_launch();
}

int mv_offset_rmsnorm_gather(const float* x, int64_t ldx, const int32_t* idx, const float* w, float eps, void* out,
                             int64_t ldo, int rows, int n, int f32, mv_stream_t stream) {
    return mv_rmsnorm_gather(x, ldx, idx, w, eps, 1.0f, out, ldo, rows, n, f32, stream);
}

int mv_rmsnorm_gather(const float* x, int64_t ldx, const int32_t* idx, const float* w, float eps, float offset,
                      void* out, int64_t ldo, int rows, int n, int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!x || !w || !out || ldx < n || ldo < n) return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    if (f32) hipLaunchKernelGGL(offset_rmsnorm_gather_kernel<true>, dim3(rows), dim3(256), 0, s, x, ldx, idx, w, eps, offset, out, ldo, n);
    else hipLaunchKernelGGL(offset_rmsnorm_gather_kernel<false>, dim3(rows), dim3(256), 0, s, x, ldx, idx, w, eps, offset, out, ldo, n);
    return check_launch();
}

int mv_embed_pair(const void* table, const void* pairs, const int32_t* ids, const int32_t* prev, float* x, int64_t ldx,
                  int rows, int n, int vocab, int64_t buckets, int64_t mul_prev, int64_t mul_cur, float scale,
                  const float* norm_w, float eps, void* h, int64_t ldh, int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0 || vocab <= 0 || buckets <= 0 || buckets > 0x7fffffff || mul_prev < 0 || mul_cur < 0)
        return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!table || !pairs || !ids || !prev || !x || ldx < n || (norm_w && (!h || ldh < n))) return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    if (f32) hipLaunchKernelGGL(embed_pair_kernel<true>, dim3(rows), dim3(256), 0, s, table, pairs, ids, prev, x, ldx, n, vocab, buckets, mul_prev, mul_cur, scale, norm_w, eps, h, ldh);
    else hipLaunchKernelGGL(embed_pair_kernel<false>, dim3(rows), dim3(256), 0, s, table, pairs, ids, prev, x, ldx, n, vocab, buckets, mul_prev, mul_cur, scale, norm_w, eps, h, ldh);
    return check_launch();
}

int mv_add_rmsnorm(const float* y1, int64_t ld1, const float* y2, int64_t ld2, float* x, int64_t ldx, const float* w,
                   float eps, void* h, int64_t ldh, int rows, int n, int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!x || ldx < n || (y1 && ld1 < n) || (y2 && (!y1 || ld2 < n)) || (w && (!h || ldh < n)) || (!w && !y1))
        return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    if (f32) hipLaunchKernelGGL(add_rmsnorm_kernel<true>, dim3(rows), dim3(256), 0, s, y1, ld1, y2, ld2, x, ldx, w, eps, h, ldh, n);
    else hipLaunchKernelGGL(add_rmsnorm_kernel<false>, dim3(rows), dim3(256), 0, s, y1, ld1, y2, ld2, x, ldx, w, eps, h, ldh, n);
    return check_launch();
}

int mv_gated_act(const float* a, int64_t lda, void* out, int64_t ldo, int rows, int n, int kind, float limit,
                 float slope, int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0 || kind < 0 || kind > 2) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!a || !out || lda < 2 * (int64_t)n || ldo < n) return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    if (n % 4 == 0 && lda % 4 == 0 && ldo % 4 == 0 && aligned16(a) && aligned16(out)) {
        const dim3 grid4(rows, (n / 4 + 255) / 256);
        if (f32) hipLaunchKernelGGL(gated_act4_kernel<true>, grid4, dim3(256), 0, s, a, lda, out, ldo, n, kind, limit, slope);
        else hipLaunchKernelGGL(gated_act4_kernel<false>, grid4, dim3(256), 0, s, a, lda, out, ldo, n, kind, limit, slope);
        return check_launch();
    }
    const dim3 grid(rows, (n + 255) / 256);
    if (f32) hipLaunchKernelGGL(gated_act_kernel<true>, grid, dim3(256), 0, s, a, lda, out, ldo, n, kind, limit, slope);
    else hipLaunchKernelGGL(gated_act_kernel<false>, grid, dim3(256), 0, s, a, lda, out, ldo, n, kind, limit, slope);
    return check_launch();
}

int mv_relu_squared(const float* in, int64_t ldi, void* out, int64_t ldo, int rows, int n, int f32,
                    mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!in || !out || ldi < n || ldo < n) return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    if (n % 4 == 0 && ldi % 4 == 0 && ldo % 4 == 0 && aligned16(in) && aligned16(out)) {
        const dim3 g4(rows, (n / 4 + 255) / 256);
        if (f32) hipLaunchKernelGGL(relu_squared4_kernel<true>, g4, dim3(256), 0, s, in, ldi, out, ldo, n / 4);
        else hipLaunchKernelGGL(relu_squared4_kernel<false>, g4, dim3(256), 0, s, in, ldi, out, ldo, n / 4);
        return check_launch();
    }
    const dim3 grid(rows, (n + 255) / 256);
    if (f32) hipLaunchKernelGGL(relu_squared_kernel<true>, grid, dim3(256), 0, s, in, ldi, out, ldo, n);
    else hipLaunchKernelGGL(relu_squared_kernel<false>, grid, dim3(256), 0, s, in, ldi, out, ldo, n);
    return check_launch();
}

int mv_softcap(float* v, int64_t count, float cap, mv_stream_t stream) {
    using namespace mv;
    if (count < 0 || !(cap > 0.f)) return MV_ERR_INVALID_ARG;
    if (count == 0) return MV_OK;
    if (!v) return MV_ERR_INVALID_ARG;
    hipLaunchKernelGGL(softcap_kernel, dim3((unsigned)((count + 255) / 256)), dim3(256), 0, (hipStream_t)stream, v, count, cap);
    return check_launch();
}

#define MV_F32_LAUNCH(kern, grid, ...)                                                              \
    do {                                                                                            \
        if (f32) hipLaunchKernelGGL(kern<true>, grid, dim3(256), 0, s, __VA_ARGS__);                \
        else hipLaunchKernelGGL(kern<false>, grid, dim3(256), 0, s, __VA_ARGS__);                   \
    } while (0)

int mv_dyt_shift(const float* x, int64_t ldx, const float* w, const float* b, const float* alpha, const float* mix,
                 float* state, void* h, int64_t ldh, const int32_t* tok_row, const int32_t* row_start,
                 const int32_t* row_len, const int32_t* row_ctx, const int32_t* row_slot, int tokens, int n, int f32,
                 mv_stream_t stream) {
    using namespace mv;
    if (tokens < 0 || n <= 0) return MV_ERR_INVALID_ARG;
    if (tokens == 0) return MV_OK;
    if (!x || !w || !b || !alpha || !mix || !state || !h || !tok_row || !row_start || !row_len || !row_ctx ||
        !row_slot || ldx < n || ldh < n)
        return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    MV_F32_LAUNCH(dyt_shift_kernel, dim3(tokens, (n + 255) / 256), x, ldx, w, b, alpha, mix, state, h, ldh, tok_row, row_start, row_len,
                  row_ctx, row_slot, n);
    return check_launch();
}

int mv_dyt_gather(const float* x, int64_t ldx, const int32_t* idx, const float* w, const float* b, const float* alpha,
                  void* out, int64_t ldo, int rows, int n, int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!x || !w || !b || !alpha || !out || ldx < n || ldo < n) return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    MV_F32_LAUNCH(dyt_gather_kernel, dim3(rows, (n + 255) / 256), x, ldx, idx, w, b, alpha, out, ldo, n);
    return check_launch();
}

int mv_dyt_residual(const float* y, int64_t ldy, const float* w, const float* b, const float* alpha, float* x,
                    int64_t ldx, void* h, int64_t ldh, const float* w2, const float* b2, const float* alpha2, int rows,
                    int n, int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!y || !w || !b || !alpha || !x || ldy < n || ldx < n || (h && ldh < n)) return MV_ERR_INVALID_ARG;
    if (w2 && (!b2 || !alpha2 || !h)) return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    MV_F32_LAUNCH(dyt_residual_kernel, dim3(rows, (n + 255) / 256), y, ldy, w, b, alpha, x, ldx, h, ldh, n, w2, b2, alpha2);
    return check_launch();
}

int mv_unitnorm_residual(const float* y, int64_t ldy, const float* w, float eps, float* x, int64_t ldx, void* h,
                         int64_t ldh, int rows, int n, int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!y || !w || !x || ldy < n || ldx < n || (h && ldh < n)) return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    MV_F32_LAUNCH(unitnorm_residual_kernel, dim3(rows), y, ldy, w, eps, x, ldx, h, ldh, n);
    return check_launch();
}

int mv_rmsnorm_rows(const float* v, int64_t ld, int per, const float* w, float eps, void* out, int64_t ldo,
                    int rows, int n, int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0 || per <= 0) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!v || !w || !out || ld < (int64_t)per * n || ldo < (int64_t)per * n) return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    const int64_t total = (int64_t)rows * per;
    MV_F32_LAUNCH(rmsnorm_rows_kernel, dim3((unsigned)((total + 3) / 4)), v, ld, per, w, eps, out, ldo, total, n);
    return check_launch();
}

int mv_gelu_gate_rows(const float* a, int64_t lda, const void* table, int64_t ldt, int off, const int32_t* ids,
                      int vocab, void* out, int64_t ldo, int rows, int n, int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0 || vocab <= 0 || off < 0) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!a || !table || !ids || !out || lda < n || ldt < off + n || ldo < n) return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    MV_F32_LAUNCH(gelu_gate_rows_kernel, dim3(rows, (n + 255) / 256), a, lda, table, ldt, off, ids, vocab, out, ldo, n);
    return check_launch();
}

int mv_silu_mul(const float* a, int64_t lda, void* out, int64_t ldo, int rows, int n, int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!a || !out || lda < 2 * (int64_t)n || ldo < n) return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    const dim3 grid(rows, (n + 255) / 256);
    MV_F32_LAUNCH(silu_mul_kernel, grid, a, lda, out, ldo, n);
    return check_launch();
}

int mv_sigmoid_gate(const float* a, int64_t lda, const float* g, int64_t ldg, void* out, int64_t ldo, int rows, int n,
                    int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!a || !out || lda < n || (g && ldg < n) || ldo < n) return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    const dim3 grid(rows, (n + 255) / 256);
    MV_F32_LAUNCH(sigmoid_gate_kernel, grid, a, lda, g, ldg, out, ldo, n);
    return check_launch();
}

int mv_gated_residual_norm(const float* y, int64_t ldy, const float* g, int64_t ldg, const float* b, int mode, float* x,
                           int64_t ldx, const float* w, float eps, float offset, float* n32, int64_t ldn, void* h,
                           int64_t ldh, int rows, int n, int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0 || mode < 0 || mode > 2) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!x || ldx < n || (mode != 0 && (!y || ldy < n)) || (mode == 1 && (!g || ldg < n)) ||
        (w && !n32 && !h) || (!w && (n32 || h)) || (n32 && ldn < n) || (h && ldh < n) || (!w && mode == 0))
        return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    if (f32) hipLaunchKernelGGL(gated_residual_norm_kernel<true>, dim3(rows), dim3(256), 0, s, y, ldy, g, ldg, b, mode, x, ldx, w, eps, offset, n32, ldn, h, ldh, n);
    else hipLaunchKernelGGL(gated_residual_norm_kernel<false>, dim3(rows), dim3(256), 0, s, y, ldy, g, ldg, b, mode, x, ldx, w, eps, offset, n32, ldn, h, ldh, n);
    return check_launch();
}

int mv_cast_concat(const float* a, int64_t lda, const float* b, int64_t ldb, void* out, int64_t ldo, int rows, int n,
                   int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!a || !b || !out || lda < n || ldb < n || ldo < 2 * (int64_t)n) return MV_ERR_INVALID_ARG;
    const dim3 grid(rows, (2 * n + 255) / 256);
    hipStream_t s = (hipStream_t)stream;
    if (f32) hipLaunchKernelGGL(cast_concat_kernel<true>, grid, dim3(256), 0, s, a, lda, b, ldb, out, ldo, n);
    else hipLaunchKernelGGL(cast_concat_kernel<false>, grid, dim3(256), 0, s, a, lda, b, ldb, out, ldo, n);
    return check_launch();
}

int mv_gelu_tanh(const float* in, int64_t ldi, void* out, int64_t ldo, int rows, int n, int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!in || !out || ldi < n || ldo < n) return MV_ERR_INVALID_ARG;
    const dim3 grid(rows, (n + 255) / 256);
    hipStream_t s = (hipStream_t)stream;
    if (f32) hipLaunchKernelGGL(gelu_tanh_kernel<true>, grid, dim3(256), 0, s, in, ldi, out, ldo, n);
    else hipLaunchKernelGGL(gelu_tanh_kernel<false>, grid, dim3(256), 0, s, in, ldi, out, ldo, n);
    return check_launch();
}

int mv_scale(float* v, int64_t count, float factor, mv_stream_t stream) {
    using namespace mv;
    if (count < 0) return MV_ERR_INVALID_ARG;
    if (count == 0) return MV_OK;
    if (!v) return MV_ERR_INVALID_ARG;
    hipLaunchKernelGGL(scale_kernel, dim3((unsigned)((count + 255) / 256)), dim3(256), 0, (hipStream_t)stream, v, count,
                       factor);
    return check_launch();
}

int mv_layernorm_residual(const float* y1, int64_t ld1, const float* r1, const float* y2, int64_t ld2, const float* r2,
                          float s, const int32_t* place, const float* weights, int top, const float* w, float eps,
                          const float* next_w, float* x, int64_t ldx, void* h, int64_t ldh, int rows, int n, int f32,
                          mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!y1 || !w || !x || ld1 < n || (y2 && ld2 < n) || ldx < n || (h && ldh < n) || (next_w && !h)) return MV_ERR_INVALID_ARG;
    if (place ? (!weights || top <= 0 || r1 || r2) : (y2 ? (!r1 || !r2) : (r1 || r2))) return MV_ERR_INVALID_ARG;
    LayernormArgs a;
    a.y1 = y1; a.r1 = r1; a.y2 = y2; a.r2 = r2; a.place = place; a.wts = weights; a.w = w; a.w2 = next_w;
    a.ld1 = ld1; a.ld2 = ld2; a.ldx = ldx; a.ldh = ldh; a.s = s; a.eps = eps; a.x = x; a.h = h; a.n = n; a.top = top;
    auto al = [](const void* p) { return !p || aligned16(p); };
    const bool even = n % 4 == 0 && ld1 % 4 == 0 && ldx % 4 == 0 && (!h || ldh % 4 == 0) && (!y2 || ld2 % 4 == 0) && al(y1) &&
                      al(y2) && al(r1) && al(r2) && al(w) && al(next_w) && al(x) && al(h);
    const int vec = even ? 4 : 1;
    // a row of a short step has its workgroup to itself on a compute unit: more threads, fewer values each
    int nt = rows > 512 ? 256 : 1024;
    while (nt > 64 && n <= vec * (nt / 2)) nt /= 2;
    while (nt < 1024 && n > vec * nt * 4) nt *= 2;
    const int turns = (n + vec * nt - 1) / (vec * nt);
    hipStream_t st = (hipStream_t)stream;
#define MV_LAYERNORM(VEC_, NV_)                                                                                      \
    do {                                                                                                             \
        if (f32) hipLaunchKernelGGL((layernorm_residual_kernel<true, VEC_, NV_>), dim3(rows), dim3(nt), 0, st, a);    \
        else hipLaunchKernelGGL((layernorm_residual_kernel<false, VEC_, NV_>), dim3(rows), dim3(nt), 0, st, a);       \
    } while (0)
    if (even && turns == 1) MV_LAYERNORM(4, 1);
    else if (even && turns == 2) MV_LAYERNORM(4, 2);
    else if (even && turns <= 4) MV_LAYERNORM(4, 4);
    else if (!even && turns == 1) MV_LAYERNORM(1, 1);
    else if (!even && turns <= 4) MV_LAYERNORM(1, 4);
    else if (!even && turns <= 16) MV_LAYERNORM(1, 16);
    else return MV_ERR_UNSUPPORTED;
#undef MV_LAYERNORM
    return check_launch();
}

int mv_layernorm_gather(const float* x, int64_t ldx, const int32_t* idx, const float* w, float eps, void* out,
                        int64_t ldo, int rows, int n, int f32, mv_stream_t stream) {
    using namespace mv;
    if (rows < 0 || n <= 0) return MV_ERR_INVALID_ARG;
    if (rows == 0) return MV_OK;
    if (!x || !w || !out || ldx < n || ldo < n) return MV_ERR_INVALID_ARG;
    hipStream_t s = (hipStream_t)stream;
    if (f32) hipLaunchKernelGGL(layernorm_gather_kernel<true>, dim3(rows), dim3(256), 0, s, x, ldx, idx, w, eps, out, ldo, n);
    else hipLaunchKernelGGL(layernorm_gather_kernel<false>, dim3(rows), dim3(256), 0, s, x, ldx, idx, w, eps, out, ldo, n);
    return check_launch();
}

}  // extern "C"
