// The residual stream in several copies, a layer norm with weight and bias, and the previous token mixed into what a mixer reads.
// float32 arithmetic throughout.
//
//   tqk_streams_fill    X[t, s] = h[t] for every copy s
//   tqk_streams_step    for every token, in one pass over its copies: first (where y is given) the update of all copies from the old ones,
//                       X'[t, r] = sum_s mix[s, r] X[t, s] + out[r] y[t]; then (where `in` is given) what the next part reads,
//                       u = sum_s in[s] X'[t, s], left as it is in u_out and / or normed, (u - mean) / sqrt(var + eps) w + b, in n_out.
//                       The variance is the mean of the squared deviations from the mean (two passes over a row kept in LDS).
//   tqk_add_layer_norm  out[i] = LN(h[rows[i]] + delta[rows[i]]) (rows null: row i; h or delta may be missing; write_back: h keeps the sum);
//                       the update may be normed itself before it is added: a part's output norm, the residual sum and the next part's norm
//                       in one pass.  A norm's bias may be missing.
//   tqk_token_shift     out[t] = n[t] + (n[t - 1] - n[t]) mu, the row before a sequence's first token of the step taken from the
//                       sequence's state (zeros before its first token); `remember` (steps of one token a sequence) also leaves n[t] there
//   tqk_shift_remember  state of sequence s = n[last token the step brings of s]
//   tqk_normed_pair_sum out[t] = c (x[t] / rms(x[t]) wx + y[t] / rms(y[t]) wy)
#include "common.h"
#include "tq_kernels.h"

#define STREAMS_MAX 16

__global__ __launch_bounds__(256)
void streams_fill_kernel(const float* __restrict__ h, float* __restrict__ X, int S, int W) {
    const size_t t = blockIdx.x;
    for (int e = threadIdx.x; e < W; e += blockDim.x) {
        const float v = h[t * W + e];
        for (int s = 0; s < S; ++s) X[(t * S + s) * W + e] = v;
    }
}

// SMAX: the most copies this instance takes (the loops over the copies are unrolled up to it)
template <typename TY, typename TN, int SMAX>
__global__ __launch_bounds__(1024)
void streams_step_kernel(float* __restrict__ X, int S, const TY* __restrict__ y, const float* __restrict__ mix, const float* __restrict__ outw,
                         const float* __restrict__ in, const float* __restrict__ nw, const float* __restrict__ nb, float eps,
                         float* __restrict__ u_out, TN* __restrict__ n_out, int W) {
    extern __shared__ float row_u[];
    __shared__ float scratch[16];
    __shared__ float s_mix[STREAMS_MAX * STREAMS_MAX], s_out[STREAMS_MAX], s_in[STREAMS_MAX];
    const size_t t = blockIdx.x;
    for (int i = threadIdx.x; i < S * S && y; i += blockDim.x) s_mix[i] = mix[i];
    if (threadIdx.x < S) {
        if (y) s_out[threadIdx.x] = outw[threadIdx.x];
        if (in) s_in[threadIdx.x] = in[threadIdx.x];
    }
    __syncthreads();
    float* xr = X + t * S * W;
    float sum = 0.f;
    for (int e = threadIdx.x; e < W; e += blockDim.x) {
        float x[SMAX];
#pragma unroll
        for (int s = 0; s < SMAX; ++s) x[s] = s < S ? xr[(size_t)s * W + e] : 0.f;
        if (y) {
            const float yv = to_float(y[t * W + e]);
            float nx[SMAX];
#pragma unroll
            for (int r = 0; r < SMAX; ++r) {
                float acc = 0.f;
                if (r < S) {
#pragma unroll
                    for (int s = 0; s < SMAX; ++s)
                        if (s < S) acc = fmaf(s_mix[s * S + r], x[s], acc);
                    acc = fmaf(s_out[r], yv, acc);
                    xr[(size_t)r * W + e] = acc;
                }
                nx[r] = acc;
            }
#pragma unroll
            for (int s = 0; s < SMAX; ++s) x[s] = nx[s];
        }
        if (in) {
            float u = 0.f;
#pragma unroll
            for (int s = 0; s < SMAX; ++s)
                if (s < S) u = fmaf(s_in[s], x[s], u);
            row_u[e] = u;
            sum += u;
            if (u_out) u_out[t * W + e] = u;
        }
    }
    if (!in || !n_out) return;
    const float mean = block_sum(sum, scratch) / (float)W;
    float ss = 0.f;
    for (int e = threadIdx.x; e < W; e += blockDim.x) { const float dlt = row_u[e] - mean; ss = fmaf(dlt, dlt, ss); }
    const float inv = 1.f / sqrtf(block_sum(ss, scratch) / (float)W + eps);
    for (int e = threadIdx.x; e < W; e += blockDim.x) n_out[t * W + e] = from_float<TN>((row_u[e] - mean) * inv * nw[e] + (nb ? nb[e] : 0.f));
}

// The update of a row may be normed itself before it is added (pw given): h += (d - mean d) / sqrt(var d + peps) pw + pb.
struct LayerNormArgs {
    float* h;
    const void* delta;
    const int32_t* rows;
    const float *w, *b;
    float eps;
    const float *pw, *pb;
    float peps;
    void* out;
    int W, write_back;
    const float* sums;              // the update as the sums of a product over pieces of its K, [pieces][rows][W] (then delta is null)
    int pieces, sums_bf16;          // sums_bf16: the finished product would have been rounded to bfloat16
    long long piece_stride;
};

template <typename TD, typename TO>
__global__ __launch_bounds__(256)
void add_layer_norm_kernel(const LayerNormArgs a) {
    extern __shared__ float row_u[];
    __shared__ float scratch[4];
    const int W = a.W;
    const size_t i = blockIdx.x, r = a.rows ? (size_t)a.rows[i] : i;
    const TD* delta = (const TD*)a.delta;
    auto update = [&](int e) -> float {
        if (!a.sums) return delta ? to_float(delta[r * W + e]) : 0.f;
        float v = 0.f;
        for (int p = 0; p < a.pieces; ++p) v += a.sums[(size_t)p * a.piece_stride + r * W + e];
        return a.sums_bf16 ? to_float(from_float<bf16_t>(v)) : v;
    };
    float pmean = 0.f, pinv = 1.f;
    if (a.pw) {
        float sum = 0.f;
        for (int e = threadIdx.x; e < W; e += blockDim.x) sum += update(e);
        pmean = block_sum(sum, scratch) / (float)W;
        float ss = 0.f;
        for (int e = threadIdx.x; e < W; e += blockDim.x) { const float dlt = update(e) - pmean; ss = fmaf(dlt, dlt, ss); }
        pinv = 1.f / sqrtf(block_sum(ss, scratch) / (float)W + a.peps);
    }
    float sum = 0.f;
    for (int e = threadIdx.x; e < W; e += blockDim.x) {
        float v = a.h ? a.h[r * W + e] : 0.f;
        if (delta || a.sums) {
            float d = update(e);
            if (a.pw) d = (d - pmean) * pinv * a.pw[e] + (a.pb ? a.pb[e] : 0.f);
            v += d;
        }
        if (a.write_back && a.h) a.h[r * W + e] = v;
        row_u[e] = v;
        sum += v;
    }
    const float mean = block_sum(sum, scratch) / (float)W;
    float ss = 0.f;
    for (int e = threadIdx.x; e < W; e += blockDim.x) { const float dlt = row_u[e] - mean; ss = fmaf(dlt, dlt, ss); }
    const float inv = 1.f / sqrtf(block_sum(ss, scratch) / (float)W + a.eps);
    TO* out = (TO*)a.out;
    for (int e = threadIdx.x; e < W; e += blockDim.x) out[i * W + e] = from_float<TO>((row_u[e] - mean) * inv * a.w[e] + (a.b ? a.b[e] : 0.f));
}

// The same for rows that fall into pieces of four elements, a thread NV of them: the update and the sum stay in registers between the
// sums over the row, whose partial results meet in LDS behind one barrier each.
__device__ __forceinline__ void load4(const float* p, float (&v)[4]) {
    const float4 x = *reinterpret_cast<const float4*>(p);
    v[0] = x.x; v[1] = x.y; v[2] = x.z; v[3] = x.w;
}
__device__ __forceinline__ void load4(const bf16_t* p, float (&v)[4]) {
    const uint2 x = *reinterpret_cast<const uint2*>(p);
    v[0] = __uint_as_float(x.x << 16); v[1] = __uint_as_float(x.x & 0xffff0000u);
    v[2] = __uint_as_float(x.y << 16); v[3] = __uint_as_float(x.y & 0xffff0000u);
}
__device__ __forceinline__ void store4(float* p, const float (&v)[4]) { *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]); }
__device__ __forceinline__ void store4(bf16_t* p, const float (&v)[4]) {
    *reinterpret_cast<uint2*>(p) = make_uint2((uint32_t)float_to_bf16_bits(v[0]) | ((uint32_t)float_to_bf16_bits(v[1]) << 16),
                                              (uint32_t)float_to_bf16_bits(v[2]) | ((uint32_t)float_to_bf16_bits(v[3]) << 16));
}
// (slots: a place of its own for every sum of the kernel, so that one barrier is enough)
__device__ __forceinline__ float row_sum(float v, float* slots) {
    v = wave_sum(v);
    if ((threadIdx.x & (TQK_WAVE - 1)) == 0) slots[threadIdx.x / TQK_WAVE] = v;
    __syncthreads();
    float total = 0.f;
    for (int w = 0; w < (int)(blockDim.x / TQK_WAVE); ++w) total += slots[w];
    return total;
}

template <typename TD, typename TO, int NV>
__global__ __launch_bounds__(1024)
void add_layer_norm_vec_kernel(const LayerNormArgs a) {
    __shared__ float slots[4][16];
    const int W = a.W, n4 = W / 4;
    const size_t i = blockIdx.x, r = a.rows ? (size_t)a.rows[i] : i;
    const TD* delta = a.delta ? (const TD*)a.delta + r * W : nullptr;
    float* h = a.h ? a.h + r * W : nullptr;
    float d[NV][4], x[NV][4];
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int c = threadIdx.x + k * blockDim.x;
#pragma unroll
        for (int j = 0; j < 4; ++j) d[k][j] = x[k][j] = 0.f;
        if (c < n4) {
            if (delta) load4(delta + 4 * c, d[k]);
            if (a.sums) {
                for (int p = 0; p < a.pieces; ++p) {
                    float v[4];
                    load4(a.sums + (size_t)p * a.piece_stride + r * W + 4 * c, v);
#pragma unroll
                    for (int j = 0; j < 4; ++j) d[k][j] += v[j];
                }
                if (a.sums_bf16) {
#pragma unroll
                    for (int j = 0; j < 4; ++j) d[k][j] = to_float(from_float<bf16_t>(d[k][j]));
                }
            }
            if (h) load4(h + 4 * c, x[k]);
        }
    }
    if (a.pw) {
        float sum = 0.f;
#pragma unroll
        for (int k = 0; k < NV; ++k)
#pragma unroll
            for (int j = 0; j < 4; ++j) sum += d[k][j];
        const float mean = row_sum(sum, slots[0]) / (float)W;
        float ss = 0.f;
#pragma unroll
        for (int k = 0; k < NV; ++k)
            if (threadIdx.x + k * blockDim.x < n4) {
#pragma unroll
                for (int j = 0; j < 4; ++j) { const float dlt = d[k][j] - mean; ss = fmaf(dlt, dlt, ss); }
            }
        const float inv = 1.f / sqrtf(row_sum(ss, slots[1]) / (float)W + a.peps);
#pragma unroll
        for (int k = 0; k < NV; ++k) {
            const int c = threadIdx.x + k * blockDim.x;
            if (c >= n4) continue;
            float w4[4], b4[4] = {0.f, 0.f, 0.f, 0.f};
            load4(a.pw + 4 * c, w4);
            if (a.pb) load4(a.pb + 4 * c, b4);
#pragma unroll
            for (int j = 0; j < 4; ++j) d[k][j] = (d[k][j] - mean) * inv * w4[j] + b4[j];
        }
    }
    float sum = 0.f;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int c = threadIdx.x + k * blockDim.x;
#pragma unroll
        for (int j = 0; j < 4; ++j) { x[k][j] += d[k][j]; sum += x[k][j]; }
        if (c < n4 && a.write_back && h) store4(h + 4 * c, x[k]);
    }
    const float mean = row_sum(sum, slots[2]) / (float)W;
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < NV; ++k)
        if (threadIdx.x + k * blockDim.x < n4) {
#pragma unroll
            for (int j = 0; j < 4; ++j) { const float dlt = x[k][j] - mean; ss = fmaf(dlt, dlt, ss); }
        }
    const float inv = 1.f / sqrtf(row_sum(ss, slots[3]) / (float)W + a.eps);
    TO* out = (TO*)a.out + i * W;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int c = threadIdx.x + k * blockDim.x;
        if (c >= n4) continue;
        float w4[4], b4[4] = {0.f, 0.f, 0.f, 0.f}, y[4];
        load4(a.w + 4 * c, w4);
        if (a.b) load4(a.b + 4 * c, b4);
#pragma unroll
        for (int j = 0; j < 4; ++j) y[j] = (x[k][j] - mean) * inv * w4[j] + b4[j];
        store4(out + 4 * c, y);
    }
}

template <typename TO>
__global__ __launch_bounds__(256)
void token_shift_kernel(const float* __restrict__ n, const float* __restrict__ mu, float* __restrict__ state, long long state_stride,
                        const int32_t* __restrict__ tok_seq, const int32_t* __restrict__ tok_pos, const int32_t* __restrict__ seq_start,
                        const int32_t* __restrict__ seq_slot, TO* __restrict__ out, int W, int remember) {
    const size_t t = blockIdx.x;
    const int seq = tok_seq[t];
    const bool inside = tok_pos[t] > seq_start[seq];
    float* st = state + (size_t)seq_slot[seq] * state_stride;
    for (int e = threadIdx.x; e < W; e += blockDim.x) {
        const float cur = n[t * W + e];
        const float prev = inside ? n[(t - 1) * W + e] : st[e];
        out[t * W + e] = from_float<TO>(cur + (prev - cur) * mu[e]);
        if (remember) st[e] = cur;
    }
}

__global__ __launch_bounds__(256)
void shift_remember_kernel(const float* __restrict__ n, float* __restrict__ state, long long state_stride, const int32_t* __restrict__ cu,
                           const int32_t* __restrict__ seq_new, const int32_t* __restrict__ seq_slot, int W) {
    const int s = blockIdx.x;
    if (seq_new[s] <= 0) return;
    const size_t t = (size_t)cu[s] + seq_new[s] - 1;
    float* st = state + (size_t)seq_slot[s] * state_stride;
    for (int e = threadIdx.x; e < W; e += blockDim.x) st[e] = n[t * W + e];
}

extern "C" int tqk_streams_max(void) { return STREAMS_MAX; }

extern "C" int tqk_streams_fill(const float* h, float* X, int n_streams, int n_tokens, int width, void* stream) {
    TQK_REQUIRE(h && X, "tqk_streams_fill: null pointer");
    TQK_REQUIRE(n_tokens >= 0 && n_streams > 0 && width > 0, "tqk_streams_fill: bad sizes");
    if (n_tokens == 0) return 0;
    streams_fill_kernel<<<n_tokens, 256, 0, (hipStream_t)stream>>>(h, X, n_streams, width);
    return tqk_check_launch("tqk_streams_fill");
}

extern "C" int tqk_streams_step(float* X, int n_streams, const void* y, int y_dtype, const float* mix, const float* out_w, const float* in_w,
                                const float* norm_w, const float* norm_b, float eps, float* u_out, void* n_out, int n_dtype, int n_tokens, int width,
                                int wide, void* stream) {
    TQK_REQUIRE(X, "tqk_streams_step: null pointer");
    TQK_REQUIRE(n_streams > 0 && n_streams <= STREAMS_MAX, "tqk_streams_step: %d copies of the stream, the kernel takes up to %d", n_streams, STREAMS_MAX);
    TQK_REQUIRE(!y || (mix && out_w), "tqk_streams_step: an update without its weights");
    TQK_REQUIRE(!n_out || (in_w && norm_w), "tqk_streams_step: a norm without its weights");
    TQK_REQUIRE(!u_out || in_w, "tqk_streams_step: a sum without its weights");
    TQK_REQUIRE(n_tokens >= 0 && width > 0 && width <= 12288, "tqk_streams_step: bad sizes");
    if (n_tokens == 0 || (!y && !in_w)) return 0;
    hipStream_t s = (hipStream_t)stream;
    const size_t lds = (size_t)width * sizeof(float);
    // wide (steps of few tokens, where the caller does not need one order of a row's sums for every kind of step): four times the
    // threads a row, so that a thread has a quarter of the loads to wait for one after the other
    const int threads = wide && width >= 1024 ? 1024 : 256;
#define TQK_SS_N(TY, TN, SMAX) streams_step_kernel<TY, TN, SMAX><<<n_tokens, threads, lds, s>>>(X, n_streams, (const TY*)y, mix, out_w, in_w, norm_w, norm_b, eps, u_out, (TN*)n_out, width)
#define TQK_SS(TY, TN) do { if (n_streams <= 1) TQK_SS_N(TY, TN, 1); else if (n_streams <= 2) TQK_SS_N(TY, TN, 2); else if (n_streams <= 4) TQK_SS_N(TY, TN, 4); \
        else if (n_streams <= 8) TQK_SS_N(TY, TN, 8); else TQK_SS_N(TY, TN, STREAMS_MAX); } while (0)
    const int yd = y ? y_dtype : TQK_F32, nd = n_out ? n_dtype : TQK_F32;
    if (yd == TQK_F32 && nd == TQK_F32) TQK_SS(float, float);
    else if (yd == TQK_F32 && nd == TQK_BF16) TQK_SS(float, bf16_t);
    else if (yd == TQK_BF16 && nd == TQK_F32) TQK_SS(bf16_t, float);
    else if (yd == TQK_BF16 && nd == TQK_BF16) TQK_SS(bf16_t, bf16_t);
    else return tqk_fail("tqk_streams_step: unknown dtypes %d, %d", y_dtype, n_dtype);
#undef TQK_SS
#undef TQK_SS_N
    return tqk_check_launch("tqk_streams_step");
}

extern "C" int tqk_add_layer_norm(float* h, const void* delta, int delta_dtype, const int32_t* rows, int n_rows, const float* weight, const float* bias,
                                  float eps, const float* delta_weight, const float* delta_bias, float delta_eps, void* out, int out_dtype, int width,
                                  int write_back, void* stream) {
    return tqk_add_layer_norm_sums(h, delta, delta_dtype, nullptr, 0, 0, rows, n_rows, weight, bias, eps, delta_weight, delta_bias, delta_eps, out, out_dtype, width,
                                   write_back, stream);
}

extern "C" int tqk_add_layer_norm_sums(float* h, const void* delta, int delta_dtype, const float* sums, int pieces, int sum_rows, const int32_t* rows, int n_rows,
                                       const float* weight, const float* bias, float eps, const float* delta_weight, const float* delta_bias, float delta_eps,
                                       void* out, int out_dtype, int width, int write_back, void* stream) {
    TQK_REQUIRE(!sums || (!delta && pieces > 0 && sum_rows > 0 && (rows || sum_rows == n_rows)), "tqk_add_layer_norm: sums of %d pieces of %d rows", pieces, sum_rows);
    TQK_REQUIRE((h || delta) && weight && out, "tqk_add_layer_norm: null pointer");
    TQK_REQUIRE(n_rows >= 0 && width > 0 && width <= 12288, "tqk_add_layer_norm: bad sizes");
    TQK_REQUIRE(!(write_back && rows), "tqk_add_layer_norm: chosen rows are not written back");
    TQK_REQUIRE(!delta_weight || delta || sums, "tqk_add_layer_norm: a norm of an update that is not there");
    if (n_rows == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    const LayerNormArgs a = {h, delta, rows, weight, bias, eps, delta_weight, delta_bias, delta_eps, out, width, write_back, sums, pieces, delta_dtype == TQK_BF16,
                             (long long)sum_rows * width};
    const int dd = delta ? delta_dtype : TQK_F32;
    TQK_REQUIRE((dd == TQK_F32 || dd == TQK_BF16) && (out_dtype == TQK_F32 || out_dtype == TQK_BF16), "tqk_add_layer_norm: unknown dtypes %d, %d", delta_dtype, out_dtype);
    const uintptr_t all = (uintptr_t)h | (uintptr_t)delta | (uintptr_t)weight | (uintptr_t)bias | (uintptr_t)delta_weight | (uintptr_t)delta_bias | (uintptr_t)out |
                          (uintptr_t)sums;
    const bool vec = width % 4 == 0 && (all & 15) == 0;
    const size_t lds = (size_t)width * sizeof(float);
    // threads by the width alone, so that a row's sums have one order whatever the step holds
    int threads = (width / 4 + TQK_WAVE - 1) / TQK_WAVE * TQK_WAVE;
    threads = threads < TQK_WAVE ? TQK_WAVE : threads > 1024 ? 1024 : threads;
    const int nv = (width / 4 + threads - 1) / threads;
#define TQK_ALN(TD, TO) do { if (!vec) add_layer_norm_kernel<TD, TO><<<n_rows, 256, lds, s>>>(a); \
        else if (nv <= 1) add_layer_norm_vec_kernel<TD, TO, 1><<<n_rows, threads, 0, s>>>(a); \
        else if (nv <= 2) add_layer_norm_vec_kernel<TD, TO, 2><<<n_rows, threads, 0, s>>>(a); \
        else add_layer_norm_vec_kernel<TD, TO, 3><<<n_rows, threads, 0, s>>>(a); } while (0)
    if (dd == TQK_F32 && out_dtype == TQK_F32) TQK_ALN(float, float);
    else if (dd == TQK_F32) TQK_ALN(float, bf16_t);
    else if (out_dtype == TQK_F32) TQK_ALN(bf16_t, float);
    else TQK_ALN(bf16_t, bf16_t);
#undef TQK_ALN
    return tqk_check_launch("tqk_add_layer_norm");
}

extern "C" int tqk_token_shift(const float* n, const float* mu, float* state, long long state_stride, const int32_t* tok_seq, const int32_t* tok_pos,
                               const int32_t* seq_start, const int32_t* seq_slot, void* out, int out_dtype, int n_tokens, int width, int remember,
                               void* stream) {
    TQK_REQUIRE(n && mu && state && tok_seq && tok_pos && seq_start && seq_slot && out, "tqk_token_shift: null pointer");
    TQK_REQUIRE(n_tokens >= 0 && width > 0 && state_stride >= width, "tqk_token_shift: bad sizes");
    if (n_tokens == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    if (out_dtype == TQK_F32) token_shift_kernel<float><<<n_tokens, 256, 0, s>>>(n, mu, state, state_stride, tok_seq, tok_pos, seq_start, seq_slot, (float*)out, width, remember);
    else if (out_dtype == TQK_BF16) token_shift_kernel<bf16_t><<<n_tokens, 256, 0, s>>>(n, mu, state, state_stride, tok_seq, tok_pos, seq_start, seq_slot, (bf16_t*)out, width, remember);
    else return tqk_fail("tqk_token_shift: unknown dtype %d", out_dtype);
    return tqk_check_launch("tqk_token_shift");
}

extern "C" int tqk_shift_remember(const float* n, float* state, long long state_stride, const int32_t* cu, const int32_t* seq_new, const int32_t* seq_slot,
                                  int n_seqs, int width, void* stream) {
    TQK_REQUIRE(n && state && cu && seq_new && seq_slot, "tqk_shift_remember: null pointer");
    TQK_REQUIRE(n_seqs >= 0 && width > 0 && state_stride >= width, "tqk_shift_remember: bad sizes");
    if (n_seqs == 0) return 0;
    shift_remember_kernel<<<n_seqs, 256, 0, (hipStream_t)stream>>>(n, state, state_stride, cu, seq_new, seq_slot, width);
    return tqk_check_launch("tqk_shift_remember");
}

// out[t] = c (x[t] / rms(x[t]) wx + y[t] / rms(y[t]) wy): the outputs of two parts that ran side by side, each normed over the row
template <typename TA, typename TO>
__global__ __launch_bounds__(256)
void normed_pair_sum_kernel(const TA* __restrict__ x, const TA* __restrict__ y, const float* __restrict__ wx, const float* __restrict__ wy, float eps,
                            float c, TO* __restrict__ out, int W) {
    __shared__ float scratch[4];
    const size_t t = blockIdx.x;
    float sx = 0.f, sy = 0.f;
    for (int e = threadIdx.x; e < W; e += blockDim.x) {
        const float a = to_float(x[t * W + e]), b = to_float(y[t * W + e]);
        sx = fmaf(a, a, sx);
        sy = fmaf(b, b, sy);
    }
    const float ix = 1.f / sqrtf(block_sum(sx, scratch) / (float)W + eps);
    const float iy = 1.f / sqrtf(block_sum(sy, scratch) / (float)W + eps);
    for (int e = threadIdx.x; e < W; e += blockDim.x)
        out[t * W + e] = from_float<TO>(c * (to_float(x[t * W + e]) * ix * wx[e] + to_float(y[t * W + e]) * iy * wy[e]));
}

extern "C" int tqk_normed_pair_sum(const void* x, const void* y, int dtype, const float* wx, const float* wy, float eps, float c, void* out, int out_dtype,
                                   int n_tokens, int width, void* stream) {
    TQK_REQUIRE(x && y && wx && wy && out, "tqk_normed_pair_sum: null pointer");
    TQK_REQUIRE(n_tokens >= 0 && width > 0, "tqk_normed_pair_sum: bad sizes");
    if (n_tokens == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
#define TQK_NPS(TA, TO) normed_pair_sum_kernel<TA, TO><<<n_tokens, 256, 0, s>>>((const TA*)x, (const TA*)y, wx, wy, eps, c, (TO*)out, width)
    if (dtype == TQK_F32 && out_dtype == TQK_F32) TQK_NPS(float, float);
    else if (dtype == TQK_BF16 && out_dtype == TQK_BF16) TQK_NPS(bf16_t, bf16_t);
    else if (dtype == TQK_BF16 && out_dtype == TQK_F32) TQK_NPS(bf16_t, float);
    else if (dtype == TQK_F32 && out_dtype == TQK_BF16) TQK_NPS(float, bf16_t);
    else return tqk_fail("tqk_normed_pair_sum: unknown dtypes %d, %d", dtype, out_dtype);
#undef TQK_NPS
    return tqk_check_launch("tqk_normed_pair_sum");
}
