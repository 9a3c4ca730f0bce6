// What time mixing puts in front of its recurrence (the recurrence itself is tqk_linear_attention with a decay of its own per key channel and
// token, and a bonus; in steps of many tokens decay_chunks.hip).
//
//   tqk_token_mixes     out[s][t] = x[t] + (x[t - 1] - x[t]) mu[s]: what each of the products that follow reads.  The row before a sequence's
//                       first token of the step comes from the sequence's state (zeros before its first token); `remember` (steps of one
//                       token a sequence) also leaves x[t] there
//   tqk_rows_remember   state of sequence s = x[last token the step brings of s]
//   tqk_low_rank_decay  log_decay[t, c] = -exp(sum_r w2[r, c] tanh(low[t, r]) + bias[c]), the logarithm of the decay
//
// float32 arithmetic; what comes and goes in the activation type is rounded once.
#include "common.h"
#include "tq_kernels.h"

#define TM_MAX_MIXES 8
#define TM_MAX_RANK 1024

// VEC neighbouring elements a thread: 8 where rows fall into such pieces (bfloat16: 16 bytes), else 1
template <typename T, int VEC> __device__ __forceinline__ void load_piece(const T* p, float* v) {
    if constexpr (VEC == 8 && sizeof(T) == 2) {
        const uint4 raw = *reinterpret_cast<const uint4*>(p);
        const uint32_t u[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
        for (int j = 0; j < 4; ++j) { v[2 * j] = __uint_as_float(u[j] << 16); v[2 * j + 1] = __uint_as_float(u[j] & 0xffff0000u); }
    } else if constexpr (VEC == 8) {
        const float4 a = reinterpret_cast<const float4*>(p)[0], b = reinterpret_cast<const float4*>(p)[1];
        v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
    } else v[0] = to_float(p[0]);
}
template <typename T, int VEC> __device__ __forceinline__ void store_piece(T* p, const float* v) {
    if constexpr (VEC == 8 && sizeof(T) == 2) {
        uint32_t u[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) u[j] = float_to_bf16_bits(v[2 * j]) | ((uint32_t)float_to_bf16_bits(v[2 * j + 1]) << 16);
        *reinterpret_cast<uint4*>(p) = make_uint4(u[0], u[1], u[2], u[3]);
    } else if constexpr (VEC == 8) {
        reinterpret_cast<float4*>(p)[0] = make_float4(v[0], v[1], v[2], v[3]);
        reinterpret_cast<float4*>(p)[1] = make_float4(v[4], v[5], v[6], v[7]);
    } else p[0] = from_float<T>(v[0]);
}

template <typename T, int VEC>
__global__ __launch_bounds__(256)
void token_mixes_kernel(const T* __restrict__ x, const float* __restrict__ mu, int n_mixes, float* __restrict__ state, long long state_stride,
                        const int32_t* __restrict__ tok_seq, const int32_t* __restrict__ tok_pos, const int32_t* __restrict__ seq_start,
                        const int32_t* __restrict__ seq_slot, T* __restrict__ out, long long mix_stride, int W, int remember) {
    const size_t t = blockIdx.x;
    const int e = (blockIdx.y * blockDim.x + threadIdx.x) * VEC;
    if (e >= W) return;
    const int seq = tok_seq[t];
    const bool inside = tok_pos[t] > seq_start[seq];
    float* st = state + (size_t)seq_slot[seq] * state_stride + e;
    float cur[VEC], prev[VEC];
    load_piece<T, VEC>(x + t * W + e, cur);
    if (inside) load_piece<T, VEC>(x + (t - 1) * W + e, prev);
    else {
#pragma unroll
        for (int j = 0; j < VEC; ++j) prev[j] = st[j];
    }
    if (remember) {
#pragma unroll
        for (int j = 0; j < VEC; ++j) st[j] = cur[j];
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) prev[j] -= cur[j];
    for (int s = 0; s < n_mixes; ++s) {
        float m[VEC], v[VEC];
        load_piece<float, VEC>(mu + (size_t)s * W + e, m);
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] = fmaf(prev[j], m[j], cur[j]);
        store_piece<T, VEC>(out + (size_t)s * mix_stride + t * W + e, v);
    }
}

template <typename T>
__global__ __launch_bounds__(256)
void rows_remember_kernel(const T* __restrict__ x, float* __restrict__ state, long long state_stride, const int32_t* __restrict__ cu,
                          const int32_t* __restrict__ seq_new, const int32_t* __restrict__ seq_slot, int W) {
    const int s = blockIdx.y;
    const int e = blockIdx.x * blockDim.x + threadIdx.x;
    if (e >= W || seq_new[s] <= 0) return;
    const size_t t = (size_t)cu[s] + seq_new[s] - 1;
    state[(size_t)seq_slot[s] * state_stride + e] = to_float(x[t * W + e]);
}

// A block takes TT tokens and CH blockDim.x channels, a thread CH channels (blockDim.x apart) of all of them; tanh(low) of the block's tokens lies in
// LDS, [rank][TT].  A decay's sum runs over the rank in order, whatever the step holds.
template <int TT, int CH>
__global__ __launch_bounds__(256)
void low_rank_decay_kernel(const float* __restrict__ low, const float* __restrict__ w2, const float* __restrict__ bias, float* __restrict__ log_decay,
                           int n_tokens, int rank, int channels) {
    extern __shared__ __attribute__((aligned(16))) float tanh_low[];
    const int t0 = blockIdx.y * TT, nt = min(TT, n_tokens - t0);
    for (int i = threadIdx.x; i < rank * TT; i += blockDim.x) {
        const int r = i / TT, tt = i % TT;
        tanh_low[i] = tt < nt ? tanhf(low[(size_t)(t0 + tt) * rank + r]) : 0.f;
    }
    __syncthreads();
    const int c0 = blockIdx.x * CH * blockDim.x + threadIdx.x;
    int c[CH];
#pragma unroll
    for (int k = 0; k < CH; ++k) c[k] = min(c0 + k * (int)blockDim.x, channels - 1);
    float acc[CH][TT];
#pragma unroll
    for (int k = 0; k < CH; ++k)
#pragma unroll
        for (int tt = 0; tt < TT; ++tt) acc[k][tt] = 0.f;
#pragma unroll 4
    for (int r = 0; r < rank; ++r) {
        float w[CH];
#pragma unroll
        for (int k = 0; k < CH; ++k) w[k] = w2[(size_t)r * channels + c[k]];
#pragma unroll
        for (int tt = 0; tt < TT; tt += 4) {
            const float4 z = *reinterpret_cast<const float4*>(tanh_low + r * TT + tt);
#pragma unroll
            for (int k = 0; k < CH; ++k) {
                acc[k][tt] = fmaf(w[k], z.x, acc[k][tt]);
                acc[k][tt + 1] = fmaf(w[k], z.y, acc[k][tt + 1]);
                acc[k][tt + 2] = fmaf(w[k], z.z, acc[k][tt + 2]);
                acc[k][tt + 3] = fmaf(w[k], z.w, acc[k][tt + 3]);
            }
        }
    }
#pragma unroll
    for (int k = 0; k < CH; ++k) {
        if (c0 + k * (int)blockDim.x >= channels) continue;
        const float b = bias[c[k]];
#pragma unroll
        for (int tt = 0; tt < TT; ++tt)
            if (tt < nt) log_decay[(size_t)(t0 + tt) * channels + c[k]] = -expf(acc[k][tt] + b);
    }
}

// The same on the matrix cores, for a second matrix w2 [channels, rank] of bfloat16 numbers (which go in exactly; tanh(low) goes in as the sum of two).
// v_mfma_f32_16x16x32_bf16: A a tile of 16 channels, B 16 tokens, so a lane holds four neighbouring channels of one token.  A block of four
// waves takes 16 tokens and 64 `tiles` channels.
typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 tm_bf16x8_t;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float tm_floatx4_t;
#define TM_MAX_CORE_RANK 256
template <int KB>
__global__ __launch_bounds__(256)
void low_rank_decay_mfma_kernel(const float* __restrict__ low, const bf16_t* __restrict__ w2, const float* __restrict__ bias, float* __restrict__ log_decay,
                                int n_tokens, int rank, int channels, int tiles) {
    __shared__ __attribute__((aligned(16))) uint2 hi_half[KB * TQK_WAVE * 2], lo_half[KB * TQK_WAVE * 2];       // tanh(low) in the lanes' order: [32 of the rank][lane][half of its eight]
    const int wave = threadIdx.x / TQK_WAVE, lane = threadIdx.x % TQK_WAVE;
    const int g = lane / 16, r = lane % 16;
    for (int i = threadIdx.x; i < KB * TQK_WAVE * 2; i += 256) {
        const int ln = i / 2 % TQK_WAVE, e0 = 32 * (i / (2 * TQK_WAVE)) + 8 * (ln / 16) + 4 * (i % 2);
        const float4 a = *reinterpret_cast<const float4*>(low + (size_t)min(blockIdx.y * 16 + ln % 16, n_tokens - 1) * rank + (e0 < rank ? e0 : 0));
        const float z[4] = {a.x, a.y, a.z, a.w};
        uint32_t hi[4], lo[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const float y = e0 < rank ? tanhf(z[e]) : 0.f;
            hi[e] = float_to_bf16_bits(y);
            lo[e] = float_to_bf16_bits(y - __uint_as_float(hi[e] << 16));
        }
        hi_half[i] = make_uint2(hi[0] | hi[1] << 16, hi[2] | hi[3] << 16);
        lo_half[i] = make_uint2(lo[0] | lo[1] << 16, lo[2] | lo[3] << 16);
    }
    __syncthreads();
    tm_bf16x8_t hi[KB], lo[KB];
#pragma unroll
    for (int kb = 0; kb < KB; ++kb) {
        hi[kb] = *reinterpret_cast<const tm_bf16x8_t*>(hi_half + (kb * TQK_WAVE + lane) * 2);
        lo[kb] = *reinterpret_cast<const tm_bf16x8_t*>(lo_half + (kb * TQK_WAVE + lane) * 2);
    }
    const int t = blockIdx.y * 16 + r, first = (blockIdx.x * tiles * 4 + wave) * 16;
    auto weights = [&](int c0, tm_bf16x8_t (&w)[KB]) {
        const bf16_t* wr = w2 + (size_t)min(c0 + r, channels - 1) * rank;
#pragma unroll
        for (int kb = 0; kb < KB; ++kb) {
            const int e0 = 32 * kb + 8 * g;
            w[kb] = *reinterpret_cast<const tm_bf16x8_t*>(wr + (e0 < rank ? e0 : 0));     // (beyond the rank tanh(low) is zero)
        }
    };
    tm_bf16x8_t w[KB], ahead[KB];
    weights(first, w);
    for (int j = 0; j < tiles; ++j) {
        const int c0 = first + 64 * j;
        if (c0 >= channels) break;
        if (j + 1 < tiles) weights(c0 + 64, ahead);
        tm_floatx4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kb = 0; kb < KB; ++kb) {
            acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[kb], hi[kb], acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[kb], lo[kb], acc, 0, 0, 0);
        }
        const int c = c0 + 4 * g;
        if (t < n_tokens && c < channels) {                 // (channels: a multiple of four)
            const float4 b = *reinterpret_cast<const float4*>(bias + c);
            *reinterpret_cast<float4*>(log_decay + (size_t)t * channels + c) = make_float4(-expf(acc[0] + b.x), -expf(acc[1] + b.y), -expf(acc[2] + b.z), -expf(acc[3] + b.w));
        }
#pragma unroll
        for (int kb = 0; kb < KB; ++kb) w[kb] = ahead[kb];
    }
}

extern "C" int tqk_low_rank_mfma_supported(int rank, int channels) { return rank > 0 && rank % 8 == 0 && rank <= TM_MAX_CORE_RANK && channels > 0 && channels % 4 == 0; }

extern "C" int tqk_low_rank_decay_mfma(const float* low, const void* w2, const float* bias, float* log_decay, int n_tokens, int rank, int channels, void* stream) {
    TQK_REQUIRE(low && w2 && bias && log_decay, "tqk_low_rank_decay_mfma: null pointer");
    TQK_REQUIRE(n_tokens >= 0 && tqk_low_rank_mfma_supported(rank, channels), "tqk_low_rank_decay_mfma: rank %d and %d channels are not taken", rank, channels);
    TQK_REQUIRE((((uintptr_t)low | (uintptr_t)w2 | (uintptr_t)bias | (uintptr_t)log_decay) & 15) == 0, "tqk_low_rank_decay_mfma: operands must be 16-byte aligned");
    if (n_tokens == 0) return 0;
    const int token_tiles = (n_tokens + 15) / 16, channel_blocks = (channels + 63) / 64;
    TQK_REQUIRE(token_tiles <= 65535, "tqk_low_rank_decay_mfma: %d tokens are more than the grid takes", n_tokens);
    // few tokens: a block per 64 channels; many: a block keeps its tokens' numbers for up to eight times as many
    int tiles = 1;
    while (tiles < 8 && (long long)token_tiles * (channel_blocks / (2 * tiles)) >= 1024) tiles *= 2;
    dim3 grid((channel_blocks + tiles - 1) / tiles, token_tiles);
    hipStream_t s = (hipStream_t)stream;
#define TQK_LRM(KB) low_rank_decay_mfma_kernel<KB><<<grid, 256, 0, s>>>(low, (const bf16_t*)w2, bias, log_decay, n_tokens, rank, channels, tiles)
    if (rank <= 32) TQK_LRM(1); else if (rank <= 64) TQK_LRM(2); else if (rank <= 128) TQK_LRM(4); else TQK_LRM(8);
#undef TQK_LRM
    return tqk_check_launch("tqk_low_rank_decay_mfma");
}

extern "C" int tqk_token_mixes(const void* x, int dtype, const float* mu, int n_mixes, float* state, long long state_stride, const int32_t* tok_seq,
                               const int32_t* tok_pos, const int32_t* seq_start, const int32_t* seq_slot, void* out, long long mix_stride, int n_tokens,
                               int width, int remember, void* stream) {
    TQK_REQUIRE(x && mu && state && tok_seq && tok_pos && seq_start && seq_slot && out, "tqk_token_mixes: null pointer");
    TQK_REQUIRE(n_tokens >= 0 && width > 0 && state_stride >= width, "tqk_token_mixes: bad sizes");
    TQK_REQUIRE(mix_stride >= (long long)n_tokens * width, "tqk_token_mixes: the mixes overlap");
    TQK_REQUIRE(n_mixes > 0 && n_mixes <= TM_MAX_MIXES, "tqk_token_mixes: %d mixes, the kernel takes up to %d", n_mixes, TM_MAX_MIXES);
    if (n_tokens == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    const bool vec = width % 8 == 0 && mix_stride % 8 == 0 && state_stride % 4 == 0 && (((uintptr_t)x | (uintptr_t)out | (uintptr_t)mu | (uintptr_t)state) & 15) == 0;
    const int pieces = vec ? width / 8 : width;
    const int threads = pieces >= 256 ? 256 : (pieces + TQK_WAVE - 1) / TQK_WAVE * TQK_WAVE;
    dim3 grid(n_tokens, (pieces + threads - 1) / threads);
#define TQK_TM(T, VEC) token_mixes_kernel<T, VEC><<<grid, threads, 0, s>>>((const T*)x, mu, n_mixes, state, state_stride, tok_seq, tok_pos, seq_start, seq_slot, (T*)out, mix_stride, width, remember)
    if (dtype == TQK_F32) { if (vec) TQK_TM(float, 8); else TQK_TM(float, 1); }
    else if (dtype == TQK_BF16) { if (vec) TQK_TM(bf16_t, 8); else TQK_TM(bf16_t, 1); }
    else return tqk_fail("tqk_token_mixes: unknown dtype %d", dtype);
#undef TQK_TM
    return tqk_check_launch("tqk_token_mixes");
}

extern "C" int tqk_rows_remember(const void* x, int dtype, float* state, long long state_stride, const int32_t* cu, const int32_t* seq_new,
                                 const int32_t* seq_slot, int n_seqs, int width, void* stream) {
    TQK_REQUIRE(x && state && cu && seq_new && seq_slot, "tqk_rows_remember: null pointer");
    TQK_REQUIRE(n_seqs >= 0 && n_seqs <= 65535 && width > 0 && state_stride >= width, "tqk_rows_remember: bad sizes");
    if (n_seqs == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    dim3 grid((width + 255) / 256, n_seqs);
    if (dtype == TQK_F32) rows_remember_kernel<float><<<grid, 256, 0, s>>>((const float*)x, state, state_stride, cu, seq_new, seq_slot, width);
    else if (dtype == TQK_BF16) rows_remember_kernel<bf16_t><<<grid, 256, 0, s>>>((const bf16_t*)x, state, state_stride, cu, seq_new, seq_slot, width);
    else return tqk_fail("tqk_rows_remember: unknown dtype %d", dtype);
    return tqk_check_launch("tqk_rows_remember");
}

extern "C" int tqk_low_rank_max(void) { return TM_MAX_RANK; }

extern "C" int tqk_low_rank_decay(const float* low, const float* w2, const float* bias, float* log_decay, int n_tokens, int rank, int channels, void* stream) {
    TQK_REQUIRE(low && w2 && bias && log_decay, "tqk_low_rank_decay: null pointer");
    TQK_REQUIRE(n_tokens >= 0 && rank > 0 && channels > 0, "tqk_low_rank_decay: bad sizes");
    TQK_REQUIRE(rank <= TM_MAX_RANK, "tqk_low_rank_decay: a rank of %d, the kernel takes up to %d", rank, TM_MAX_RANK);
    if (n_tokens == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    if (n_tokens <= 256) {
        dim3 grid((channels + TQK_WAVE - 1) / TQK_WAVE, (n_tokens + 3) / 4);
        low_rank_decay_kernel<4, 1><<<grid, TQK_WAVE, (size_t)rank * 4 * sizeof(float), s>>>(low, w2, bias, log_decay, n_tokens, rank, channels);
    } else {
        dim3 grid((channels + 511) / 512, (n_tokens + 15) / 16);
        TQK_REQUIRE(grid.y <= 65535, "tqk_low_rank_decay: %d tokens are more than the grid takes", n_tokens);
        low_rank_decay_kernel<16, 2><<<grid, 256, (size_t)rank * 16 * sizeof(float), s>>>(low, w2, bias, log_decay, n_tokens, rank, channels);
    }
    return tqk_check_launch("tqk_low_rank_decay");
}
