// A matrix state with a decay per key channel and token, for steps that bring many tokens of a sequence: chunks of up to 64 tokens on the matrix
// cores (bfloat16 in, head sizes up to 128).
//
//   o_t = S_(t-1)^T r_t + (sum_i u_i k_ti r_ti) v_t,   S_t = diag(a_t) S_(t-1) + k_t v_t^T,   a given by its logarithm
//
//   tqk_decay_local   a chunk's own part of the state, sum_s (k_s * exp(what is left of the chunk behind s)) v_s^T, and its decay per channel;
//                     tqk_chunk_carry makes of them the state every chunk starts from
//   tqk_decay_apply   the outputs of a chunk: P V + R S with P[t, s] = sum_i r_ti k_si exp(L_(t-1),i - L_si) for s < t, the bonus on the
//                     diagonal, and R the chunk's r times what is left of the starting state; then the heads' norm, weight and gate
//
// L is the running sum of the logarithms.  An exponential of a difference of L's would overflow where it is split into two factors naively: a chunk
// is cut into four sets of 16 tokens, and between a set of t and an earlier set of s both factors are taken against the border in front of
// t's set, so that each is at most 1.  Inside a set every pair has its own exponentials.
// Every float32 operand goes in as the sum of two bfloat16 ones (the product of their small parts left out), sums are float32.
// A logarithm below -40 counts as -40: what it leaves is nothing beside anything in float32, and the running sums keep their digits.
#include "common.h"
#include "tq_kernels.h"

#define DC_CHUNK 64
#define DC_MAX_D 128
#define DC_P_NUMBERS (32 * 40 + 32 * 72)
#define DC_LOG_FLOOR -40.f
#define DC_LOG2E 1.4426950408889634f

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 dc_bf16x8_t;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float dc_floatx4_t;
union dc_pack8 {
    dc_bf16x8_t v;
    uint16_t u[8];
    uint4 q;
};
__device__ __forceinline__ float bits_float(uint32_t b) { return __uint_as_float(b << 16); }
// a float32 number as the sum of two bfloat16 ones
__device__ __forceinline__ void two_parts(float x, uint16_t& hi, uint16_t& lo) {
    hi = float_to_bf16_bits(x);
    lo = float_to_bf16_bits(x - bits_float(hi));
}
__device__ __forceinline__ dc_floatx4_t mfma(const dc_pack8& a, const dc_pack8& b, dc_floatx4_t c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.v, c, 0, 0, 0);
}

// Where row t of P begins in LDS: the first 32 tokens see 32 keys at most, the others 64; rows are 16 bytes longer than that, against bank conflicts.
__device__ __forceinline__ int p_row(int t) { return t < 32 ? 40 * t : 32 * 40 + 72 * (t - 32); }

struct DecayChunkArgs {
    const bf16_t *r, *k, *v;
    long long stride;               // elements between the rows of r, k and v (heads side by side)
    const float* log_decay;         // [tokens, heads * d]
    const float* bonus;             // [heads, d]
    const int32_t *chunk_row0, *chunk_count;
    float* chunk_state;             // [chunks][heads][d][dv]
    float* chunk_decay;             // [chunks][heads * d]
    const float* norm_w;            // [heads * dv]
    float eps;
    const bf16_t* gate;             // rows `gate_stride` apart
    long long gate_stride;
    bf16_t* out;                    // [tokens, heads * dv]
    int H, d, dv;
};

// ---- a chunk's own part of the state -----------------------------------------------------------------------
// A wave: 64 key channels by 64 columns of one head of one chunk.  Where k runs over tokens, an operand's eight numbers lie in eight rows of memory:
// a lane loads four neighbouring elements of a row at once, one for each of four tiles, so that row (or column) r of tile j is element
// 4 r + j of a group of 64.
__global__ __launch_bounds__(4 * TQK_WAVE)
void decay_local_kernel(const DecayChunkArgs a, int n_items) {
    const int wave = threadIdx.x / TQK_WAVE, lane = threadIdx.x % TQK_WAVE;
    const int item = blockIdx.x * 4 + wave;
    if (item >= n_items) return;
    const int vts = (a.dv + 63) / 64, dts = (a.d + 63) / 64;
    const int v0 = (item % vts) * 64, d0 = (item / vts % dts) * 64, head = item / (vts * dts) % a.H, chunk = item / (vts * dts * a.H);
    const int g = lane / 16, r = lane % 16;
    const long long row0 = a.chunk_row0[chunk];
    const int count = a.chunk_count[chunk];
    const bool d_in = d0 + 4 * r < a.d, v_in = v0 + 4 * r < a.dv;
    const int ch = d_in ? d0 + 4 * r : 0;
    const bf16_t* kb = a.k + (size_t)head * a.d + ch;
    const bf16_t* vb = a.v + (size_t)head * a.dv + (v_in ? v0 + 4 * r : 0);
    const float* lb = a.log_decay + (size_t)head * a.d + ch;
    const size_t l_stride = (size_t)a.H * a.d;
    uint2 kr[2][8], vr[2][8];
    float w[2][8][4];
#pragma unroll
    for (int ks = 0; ks < 2; ++ks)
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const long long row = row0 + min(32 * ks + 8 * g + e, count - 1);
            kr[ks][e] = *reinterpret_cast<const uint2*>(kb + row * a.stride);
            vr[ks][e] = *reinterpret_cast<const uint2*>(vb + row * a.stride);
            const float4 l = *reinterpret_cast<const float4*>(lb + row * l_stride);
            const bool in = 32 * ks + 8 * g + e < count;
            w[ks][e][0] = in ? fmaxf(l.x, DC_LOG_FLOOR) : 0.f; w[ks][e][1] = in ? fmaxf(l.y, DC_LOG_FLOOR) : 0.f;
            w[ks][e][2] = in ? fmaxf(l.z, DC_LOG_FLOOR) : 0.f; w[ks][e][3] = in ? fmaxf(l.w, DC_LOG_FLOOR) : 0.f;
        }
    // what is left of the chunk behind a token: the sums of the logarithms of the later tokens, in the lane's eight, then over the lanes
    float total[4];
#pragma unroll
    for (int c = 0; c < 4; ++c) {
        float seg[2];
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
            float run = 0.f;
#pragma unroll
            for (int e = 7; e >= 0; --e) {
                const float l = w[ks][e][c];
                w[ks][e][c] = run;
                run += l;
            }
            seg[ks] = run;
        }
        float later[2], all[2];
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
            const float s1 = __shfl_xor(seg[ks], 16, TQK_WAVE), s2 = __shfl_xor(seg[ks], 32, TQK_WAVE), s3 = __shfl_xor(seg[ks], 48, TQK_WAVE);
            later[ks] = ((g ^ 1) > g ? s1 : 0.f) + ((g ^ 2) > g ? s2 : 0.f) + ((g ^ 3) > g ? s3 : 0.f);
            all[ks] = (seg[ks] + s1) + (s2 + s3);
        }
        later[0] += all[1];
        total[c] = all[0] + all[1];
#pragma unroll
        for (int ks = 0; ks < 2; ++ks)
#pragma unroll
            for (int e = 0; e < 8; ++e)
                w[ks][e][c] = d_in && 32 * ks + 8 * g + e < count ? __builtin_amdgcn_exp2f((w[ks][e][c] + later[ks]) * DC_LOG2E) : 0.f;
    }
    dc_floatx4_t acc[4][4];
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int c = 0; c < 4; ++c) acc[j][c] = dc_floatx4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
        dc_pack8 hi[4], lo[4], vv[4];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const uint2 kk = kr[ks][e], vq = vr[ks][e];
            const float k4[4] = {bits_float(kk.x & 0xffff), bits_float(kk.x >> 16), bits_float(kk.y & 0xffff), bits_float(kk.y >> 16)};
#pragma unroll
            for (int j = 0; j < 4; ++j) two_parts(k4[j] * w[ks][e][j], hi[j].u[e], lo[j].u[e]);
            vv[0].u[e] = (uint16_t)vq.x; vv[1].u[e] = (uint16_t)(vq.x >> 16);
            vv[2].u[e] = (uint16_t)vq.y; vv[3].u[e] = (uint16_t)(vq.y >> 16);
        }
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
            for (int c = 0; c < 4; ++c) {
                acc[j][c] = mfma(hi[j], vv[c], acc[j][c]);
                acc[j][c] = mfma(lo[j], vv[c], acc[j][c]);
            }
    }
    float* S = a.chunk_state + ((size_t)chunk * a.H + head) * a.d * a.dv;
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int row = d0 + 4 * (4 * g + i) + j;
            if (row < a.d && v_in)
                *reinterpret_cast<float4*>(S + (size_t)row * a.dv + v0 + 4 * r) = make_float4(acc[j][0][i], acc[j][1][i], acc[j][2][i], acc[j][3][i]);
        }
    if (v0 == 0 && g == 0 && d_in)
        *reinterpret_cast<float4*>(a.chunk_decay + ((size_t)chunk * a.H + head) * a.d + ch) =
            make_float4(expf(total[0]), expf(total[1]), expf(total[2]), expf(total[3]));
}

// ---- the outputs of a chunk ----------------------------------------------------------------------------------
// A block of four waves: one head of one chunk, a wave 16 of its tokens (rows of P that no other wave reads) and all NG groups of 64 columns.
// In LDS: the running sums inside each set of 16 tokens (in units of log 2), r and k, P in two parts.
template <int NG, int KB>
__global__ __launch_bounds__(4 * TQK_WAVE)
void decay_apply_kernel(const DecayChunkArgs a) {
    extern __shared__ __attribute__((aligned(16))) unsigned char dc_lds[];
    const int d = a.d, dv = a.dv, H = a.H;
    const int ls = d + 4, rs = d + 8;                               // elements between rows: 16 bytes more than a row
    float* L = reinterpret_cast<float*>(dc_lds);                    // [64][ls]
    uint16_t* rl = reinterpret_cast<uint16_t*>(L + DC_CHUNK * ls);  // [64][rs]
    uint16_t* kl = rl + DC_CHUNK * rs;                              // [64][rs]
    uint16_t* p_hi = kl + DC_CHUNK * rs;                            // rows at p_row(t)
    uint16_t* p_lo = p_hi + DC_P_NUMBERS;
    const int wave = threadIdx.x / TQK_WAVE, lane = threadIdx.x % TQK_WAVE;
    const int g = lane / 16, r = lane % 16;
    const int head = blockIdx.x, chunk = blockIdx.y;
    const long long row0 = a.chunk_row0[chunk];
    const int count = a.chunk_count[chunk];
    // bring in: a thread one channel of one set's running sums, and pieces of eight elements of r and k
    for (int e = threadIdx.x; e < 4 * d; e += blockDim.x) {
        const int set = e / d, c = e % d;
        float run = 0.f, l[16];
#pragma unroll
        for (int t = 0; t < 16; ++t) l[t] = a.log_decay[(size_t)(row0 + min(16 * set + t, count - 1)) * H * d + (size_t)head * d + c];
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            if (16 * set + t < count) run += fmaxf(l[t], DC_LOG_FLOOR) * DC_LOG2E;
            L[(16 * set + t) * ls + c] = run;
        }
    }
    for (int e = threadIdx.x; e < DC_CHUNK * (d / 8); e += blockDim.x) {
        const int t = e / (d / 8), c = (e % (d / 8)) * 8;
        const size_t at = (size_t)(row0 + min(t, count - 1)) * a.stride + (size_t)head * d + c;
        uint4 rv = *reinterpret_cast<const uint4*>(a.r + at), kv = *reinterpret_cast<const uint4*>(a.k + at);
        if (t >= count) rv = kv = make_uint4(0, 0, 0, 0);
        *reinterpret_cast<uint4*>(rl + t * rs + c) = rv;
        *reinterpret_cast<uint4*>(kl + t * rs + c) = kv;
    }
    __syncthreads();
    const int first = 16 * wave;                                    // the wave's first token
    if (first >= count) return;

    // r of the wave's tokens (token r, channels 32 kk + 8 g ..) against the border in front of them, in two parts
    auto running = [&](int t, int e0, float* out) {                 // L of token t's set up to and with t, eight channels
        const float4 x = *reinterpret_cast<const float4*>(L + t * ls + e0), y = *reinterpret_cast<const float4*>(L + t * ls + e0 + 4);
        out[0] = x.x; out[1] = x.y; out[2] = x.z; out[3] = x.w; out[4] = y.x; out[5] = y.y; out[6] = y.z; out[7] = y.w;
    };
    auto pieces = [&](int kk, const float* more, dc_pack8& hi, dc_pack8& lo) {
        const int e0 = 32 * kk + 8 * g, e0c = e0 < d ? e0 : 0;
        float before[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
        if (r > 0) running(first + r - 1, e0c, before);
        dc_pack8 x;
        x.q = *reinterpret_cast<const uint4*>(rl + (first + r) * rs + e0c);
        if (e0 >= d) x.q = make_uint4(0, 0, 0, 0);
#pragma unroll
        for (int e = 0; e < 8; ++e) two_parts(bits_float(x.u[e]) * __builtin_amdgcn_exp2f(before[e] + (more ? more[e] : 0.f)), hi.u[e], lo.u[e]);
    };
    dc_floatx4_t s[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) s[j] = dc_floatx4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kk = 0; kk < KB; ++kk) {
        if (32 * kk >= d) continue;
        const int e0 = 32 * kk + 8 * g, e0c = e0 < d ? e0 : 0;
        dc_pack8 rh, rlo;
        pieces(kk, nullptr, rh, rlo);
        // keys of earlier sets, from the nearest back: what lies between grows by a set's whole decay
        float between[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 2; j >= 0; --j) {
            if (j >= wave) continue;
            float whole[8], upto[8];
            running(16 * j + 15, e0c, whole);
            running(16 * j + r, e0c, upto);
            dc_pack8 x, kh, klo;
            x.q = *reinterpret_cast<const uint4*>(kl + (16 * j + r) * rs + e0c);
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                two_parts(bits_float(x.u[e]) * __builtin_amdgcn_exp2f(whole[e] - upto[e] + between[e]), kh.u[e], klo.u[e]);
                between[e] += whole[e];
            }
            s[j] = mfma(kh, rh, s[j]);
            s[j] = mfma(kh, rlo, s[j]);
            s[j] = mfma(klo, rh, s[j]);
        }
    }
    // P: the earlier sets' part (a lane has token r, keys 4 g ..), zeros for the keys behind, then the set's own pairs
    {
        const int at = p_row(first + r) + 4 * g;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            if (j > (wave | 1)) continue;
            uint16_t h4[4] = {0, 0, 0, 0}, l4[4] = {0, 0, 0, 0};
            if (j < wave) {
#pragma unroll
                for (int i = 0; i < 4; ++i) two_parts(s[j][i], h4[i], l4[i]);
            }
            *reinterpret_cast<uint2*>(p_hi + at + 16 * j) = make_uint2(h4[0] | ((uint32_t)h4[1] << 16), h4[2] | ((uint32_t)h4[3] << 16));
            *reinterpret_cast<uint2*>(p_lo + at + 16 * j) = make_uint2(l4[0] | ((uint32_t)l4[1] << 16), l4[2] | ((uint32_t)l4[3] << 16));
        }
    }
    __builtin_amdgcn_wave_barrier();
    // (the pairs s < t of 16 tokens: 120, two rounds of the wave)
#pragma unroll
    for (int round = 0; round < 2; ++round) {
        const int p = lane + TQK_WAVE * round;
        if (p >= 120) continue;
        int t = (int)((1.f + sqrtf(1.f + 8.f * (float)p)) * 0.5f);
        while (t * (t - 1) / 2 > p) --t;
        while ((t + 1) * t / 2 <= p) ++t;
        const int q = p - t * (t - 1) / 2;
        const float* la = L + (first + t - 1) * ls;
        const float* lb = L + (first + q) * ls;
        const uint16_t* rr = rl + (first + t) * rs;
        const uint16_t* kr = kl + (first + q) * rs;
        float sum = 0.f;
#pragma unroll 4
        for (int c = 0; c < d; c += 4) {
            const float4 x = *reinterpret_cast<const float4*>(la + c), y = *reinterpret_cast<const float4*>(lb + c);
            const uint2 ra = *reinterpret_cast<const uint2*>(rr + c), ka = *reinterpret_cast<const uint2*>(kr + c);
            sum = fmaf(bits_float(ra.x & 0xffff) * bits_float(ka.x & 0xffff), __builtin_amdgcn_exp2f(x.x - y.x), sum);
            sum = fmaf(bits_float(ra.x >> 16) * bits_float(ka.x >> 16), __builtin_amdgcn_exp2f(x.y - y.y), sum);
            sum = fmaf(bits_float(ra.y & 0xffff) * bits_float(ka.y & 0xffff), __builtin_amdgcn_exp2f(x.z - y.z), sum);
            sum = fmaf(bits_float(ra.y >> 16) * bits_float(ka.y >> 16), __builtin_amdgcn_exp2f(x.w - y.w), sum);
        }
        two_parts(sum, p_hi[p_row(first + t) + first + q], p_lo[p_row(first + t) + first + q]);
    }
    {
        // the diagonal: the bonus, a token's channels in pieces of four dealt out to its four lanes
        const float* u = a.bonus + (size_t)head * d;
        float sum = 0.f;
        for (int c = 4 * g; c < d; c += 16) {
            const uint2 ra = *reinterpret_cast<const uint2*>(rl + (first + r) * rs + c), ka = *reinterpret_cast<const uint2*>(kl + (first + r) * rs + c);
            const float4 u4 = *reinterpret_cast<const float4*>(u + c);
            sum = fmaf(u4.x * bits_float(ka.x & 0xffff), bits_float(ra.x & 0xffff), sum);
            sum = fmaf(u4.y * bits_float(ka.x >> 16), bits_float(ra.x >> 16), sum);
            sum = fmaf(u4.z * bits_float(ka.y & 0xffff), bits_float(ra.y & 0xffff), sum);
            sum = fmaf(u4.w * bits_float(ka.y >> 16), bits_float(ra.y >> 16), sum);
        }
        sum += __shfl_xor(sum, 16, TQK_WAVE);
        sum += __shfl_xor(sum, 32, TQK_WAVE);
        if (g == 0) two_parts(sum, p_hi[p_row(first + r) + first + r], p_lo[p_row(first + r) + first + r]);
    }
    __builtin_amdgcn_wave_barrier();

    dc_floatx4_t acc[NG][4];
#pragma unroll
    for (int n = 0; n < NG; ++n)
#pragma unroll
        for (int c = 0; c < 4; ++c) acc[n][c] = dc_floatx4_t{0.f, 0.f, 0.f, 0.f};
    // what lies in the state the chunk starts from
    const float* S = a.chunk_state + ((size_t)chunk * H + head) * d * dv;
#pragma unroll
    for (int kk = 0; kk < KB; ++kk) {
        if (32 * kk >= d) continue;
        const int e0 = 32 * kk + 8 * g, e0c = e0 < d ? e0 : 0;
        float more[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < 3; ++j) {
            if (j >= wave) continue;
            float whole[8];
            running(16 * j + 15, e0c, whole);
#pragma unroll
            for (int e = 0; e < 8; ++e) more[e] += whole[e];
        }
        dc_pack8 rh, rlo;
        pieces(kk, more, rh, rlo);
#pragma unroll
        for (int n = 0; n < NG; ++n) {
            const int v0 = 64 * n + 4 * r;
            const float* Sc = S + (v0 < dv ? v0 : 0);
            dc_pack8 hi[4], lo[4];
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const float4 x = *reinterpret_cast<const float4*>(Sc + (size_t)(e0c + e) * dv);
                two_parts(x.x, hi[0].u[e], lo[0].u[e]);
                two_parts(x.y, hi[1].u[e], lo[1].u[e]);
                two_parts(x.z, hi[2].u[e], lo[2].u[e]);
                two_parts(x.w, hi[3].u[e], lo[3].u[e]);
            }
#pragma unroll
            for (int c = 0; c < 4; ++c) {
                acc[n][c] = mfma(rh, hi[c], acc[n][c]);
                acc[n][c] = mfma(rh, lo[c], acc[n][c]);
                acc[n][c] = mfma(rlo, hi[c], acc[n][c]);
            }
        }
    }
    // what the chunk's own tokens give
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
        if (32 * ks > first + 15) continue;                         // keys behind all of the wave's tokens
        dc_pack8 ph, pl;
        const int at = p_row(first + r) + 32 * ks + 8 * g;
        ph.q = *reinterpret_cast<const uint4*>(p_hi + at);
        pl.q = *reinterpret_cast<const uint4*>(p_lo + at);
#pragma unroll
        for (int n = 0; n < NG; ++n) {
            const int v0 = 64 * n + 4 * r;
            const bf16_t* vb = a.v + (size_t)head * dv + (v0 < dv ? v0 : 0);
            dc_pack8 vv[4];
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const uint2 x = *reinterpret_cast<const uint2*>(vb + (row0 + min(32 * ks + 8 * g + e, count - 1)) * a.stride);
                vv[0].u[e] = (uint16_t)x.x; vv[1].u[e] = (uint16_t)(x.x >> 16);
                vv[2].u[e] = (uint16_t)x.y; vv[3].u[e] = (uint16_t)(x.y >> 16);
            }
#pragma unroll
            for (int c = 0; c < 4; ++c) {
                acc[n][c] = mfma(ph, vv[c], acc[n][c]);
                acc[n][c] = mfma(pl, vv[c], acc[n][c]);
            }
        }
    }
    // the head's norm, its weight and the gate (a lane: tokens 4 g + i, columns 64 n + 4 r ..)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        float ss = 0.f;
#pragma unroll
        for (int n = 0; n < NG; ++n)
            if (64 * n + 4 * r < dv) {
#pragma unroll
                for (int c = 0; c < 4; ++c) ss = fmaf(acc[n][c][i], acc[n][c][i], ss);
            }
#pragma unroll
        for (int o = 1; o < 16; o <<= 1) ss += __shfl_xor(ss, o, TQK_WAVE);
        const float inv = 1.f / sqrtf(ss / (float)dv + a.eps);
        const int t = first + 4 * g + i;
        if (t >= count) continue;
#pragma unroll
        for (int n = 0; n < NG; ++n) {
            const int v0 = 64 * n + 4 * r;
            if (v0 >= dv) continue;
            const float4 w4 = *reinterpret_cast<const float4*>(a.norm_w + (size_t)head * dv + v0);
            const uint2 gq = *reinterpret_cast<const uint2*>(a.gate + (row0 + t) * a.gate_stride + (size_t)head * dv + v0);
            const float g4[4] = {bits_float(gq.x & 0xffff), bits_float(gq.x >> 16), bits_float(gq.y & 0xffff), bits_float(gq.y >> 16)};
            const float ww[4] = {w4.x, w4.y, w4.z, w4.w};
            uint16_t o4[4];
#pragma unroll
            for (int c = 0; c < 4; ++c) o4[c] = float_to_bf16_bits(acc[n][c][i] * inv * ww[c] * (g4[c] / (1.f + expf(-g4[c]))));
            *reinterpret_cast<uint2*>(a.out + ((size_t)(row0 + t) * H + head) * dv + v0) = make_uint2(o4[0] | ((uint32_t)o4[1] << 16), o4[2] | ((uint32_t)o4[3] << 16));
        }
    }
}

extern "C" int tqk_decay_chunks_supported(int d, int dv) { return d > 0 && d % 8 == 0 && d <= DC_MAX_D && dv > 0 && dv % 4 == 0 && dv <= 128; }

static int decay_chunk_args(DecayChunkArgs& a, const void* k, const void* v, long long stride, const float* log_decay, const int32_t* chunk_row0,
                            const int32_t* chunk_count, int n_chunks, float* chunk_state, int heads, int d, int dv) {
    TQK_REQUIRE(k && v && log_decay && chunk_row0 && chunk_count && chunk_state, "tqk_decay chunks: null pointer");
    TQK_REQUIRE(tqk_decay_chunks_supported(d, dv), "tqk_decay chunks: heads of %d and %d elements are not taken", d, dv);
    TQK_REQUIRE(n_chunks >= 0 && n_chunks <= 65535 && heads > 0, "tqk_decay chunks: bad sizes");
    TQK_REQUIRE(stride % 8 == 0 && ((((uintptr_t)k | (uintptr_t)chunk_state | (uintptr_t)log_decay) & 15) | ((uintptr_t)v & 7)) == 0,
                "tqk_decay chunks: rows of k and of the logarithms must begin at multiples of 16 bytes, of v at multiples of 8");
    a = {};
    a.k = (const bf16_t*)k; a.v = (const bf16_t*)v; a.stride = stride; a.log_decay = log_decay;
    a.chunk_row0 = chunk_row0; a.chunk_count = chunk_count; a.chunk_state = chunk_state;
    a.H = heads; a.d = d; a.dv = dv;
    return 0;
}

extern "C" int tqk_decay_local(const void* k, const void* v, long long stride, const float* log_decay, const int32_t* chunk_row0, const int32_t* chunk_count,
                               int n_chunks, float* chunk_state, float* chunk_decay, int heads, int d, int dv, void* stream) {
    DecayChunkArgs a;
    if (decay_chunk_args(a, k, v, stride, log_decay, chunk_row0, chunk_count, n_chunks, chunk_state, heads, d, dv)) return -1;
    TQK_REQUIRE(chunk_decay && ((uintptr_t)chunk_decay & 15) == 0, "tqk_decay_local: no place for the chunks' decays");
    a.chunk_decay = chunk_decay;
    const long long items = (long long)n_chunks * heads * ((d + 63) / 64) * ((dv + 63) / 64);
    TQK_REQUIRE(items <= 0x7fffffff, "tqk_decay_local: too many chunks");
    if (items == 0) return 0;
    decay_local_kernel<<<(unsigned)((items + 3) / 4), 4 * TQK_WAVE, 0, (hipStream_t)stream>>>(a, (int)items);
    return tqk_check_launch("tqk_decay_local");
}

extern "C" int tqk_decay_apply(const void* r, const void* k, const void* v, long long stride, const float* log_decay, const float* bonus, const int32_t* chunk_row0,
                               const int32_t* chunk_count, int n_chunks, float* chunk_state, const float* norm_weight, float eps, const void* gate,
                               long long gate_stride, void* out, int heads, int d, int dv, void* stream) {
    DecayChunkArgs a;
    if (decay_chunk_args(a, k, v, stride, log_decay, chunk_row0, chunk_count, n_chunks, chunk_state, heads, d, dv)) return -1;
    TQK_REQUIRE(r && bonus && norm_weight && gate && out, "tqk_decay_apply: null pointer");
    TQK_REQUIRE((((uintptr_t)r | (uintptr_t)bonus | (uintptr_t)norm_weight) & 15) == 0 && (((uintptr_t)gate | (uintptr_t)out) & 7) == 0 && gate_stride % 4 == 0,
                "tqk_decay_apply: operands are not aligned");
    if (n_chunks == 0) return 0;
    a.r = (const bf16_t*)r; a.bonus = bonus; a.norm_w = norm_weight; a.eps = eps; a.gate = (const bf16_t*)gate; a.gate_stride = gate_stride; a.out = (bf16_t*)out;
    const size_t lds = (size_t)DC_CHUNK * ((d + 4) * sizeof(float) + 2 * (d + 8) * sizeof(uint16_t)) + 2 * DC_P_NUMBERS * sizeof(uint16_t);
    dim3 grid(heads, n_chunks);
    hipStream_t s = (hipStream_t)stream;
#define TQK_DA(NG, KB) do { \
        if (lds > 65536) { \
            static const int grown = (int)hipFuncSetAttribute((const void*)decay_apply_kernel<NG, KB>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024); \
            TQK_REQUIRE(grown == 0, "tqk_decay_apply: the device gives a block no %zu bytes of LDS", lds); \
        } \
        decay_apply_kernel<NG, KB><<<grid, 4 * TQK_WAVE, lds, s>>>(a); } while (0)
#define TQK_DA_K(NG) do { if (d <= 32) TQK_DA(NG, 1); else if (d <= 64) TQK_DA(NG, 2); else TQK_DA(NG, 4); } while (0)
    if (dv <= 64) TQK_DA_K(1);
    else TQK_DA_K(2);
#undef TQK_DA_K
#undef TQK_DA
    return tqk_check_launch("tqk_decay_apply");
}
