// The matrix memory of an mLSTM: per head a matrix S [d][dv] and a vector n [d], both decayed and written to by one number per head and
// token each, kept as logarithms against a running maximum m so that nothing overflows.
//
//   a_t = c tanh((w_i x_t + b_i) / c),   f_t = log sigmoid(c tanh((w_f x_t + b_f) / c))
//   m_t = max(f_t + m_(t-1), a_t);   kappa_t = f_t + m_(t-1) - m_t,   tau_t = a_t - m_t         (both at most 0)
//   S_t = e^kappa S_(t-1) + e^tau k_t v_t^T,   n_t = e^kappa n_(t-1) + e^tau k_t
//   o_t = S_t^T q_t / (max(|n_t . q_t|, e^(-m_t)) + 1e-6)
//
// Everything here is float32; q, k, v come from the products.  A slot's state is [heads][d * dv (S) | d (n)], then [heads] (m).
//
//   tqk_mlstm_gates   kappa, tau and m of every token, in the tokens' order, m carried in the state; where inv_den is given also n
//                     and 1 / (the denominator of o_t).  S itself is then tqk_linear_attention's, with kappa, tau and inv_den.
//
// Steps that bring many tokens of a sequence in bfloat16 go through the matrix cores in chunks of up to 64 tokens:
//   tqk_mlstm_gate_scan   kappa, tau and m alone, 16 pieces of 64 tokens at a time (m_t = F_t + max(m_0, max_(s <= t) (a_s - F_s)) with F
//                         the running sum of f, so that pieces meet through two numbers each)
//   tqk_mlstm_local       what a chunk adds: U = sum_s e^(C_end - C_s + tau_s) k_s v_s^T and the same with k_s alone (C the running sum of
//                         kappa inside the chunk), and its decay e^C_end; between this and the next tqk_chunk_carry turns U into the state
//                         the chunk starts from
//   tqk_mlstm_apply       P_ts = q_t . k_s e^(C_t - C_s + tau_s) for s <= t;  o_t = (e^C_t S_0^T q_t + sum_s P_ts v_s) / (max(|e^C_t n_0 . q_t
//                         + sum_s P_ts|, e^(-m_t)) + 1e-6), and where a block holds a whole head, the head's norm and the output gate
// q, k and v enter the products as the bfloat16 numbers they are; what is float32 (weighted keys, states, P) enters as the sum of two
// bfloat16 numbers, which leaves 16 bits of it.
#include "common.h"
#include "tq_kernels.h"

#define ML_MAX_D 512

__device__ __forceinline__ float log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }

// A wave per (head, sequence): 64 tokens' logarithms at a time, a lane a token; then the maximum from token to token (the lanes' numbers
// are handed round in registers), and with inv_den the vector n too, its elements dealt out to the lanes, the next token's q and k asked
// for before this one's are used.
template <typename T, int NR>
__global__ __launch_bounds__(TQK_WAVE)
void mlstm_gates_kernel(const float* __restrict__ z, long long z_stride, const float* __restrict__ bias, float cap, const T* __restrict__ q,
                        const T* __restrict__ k, long long stride, float q_scale, float* __restrict__ state, long long state_stride, long long head_stride,
                        long long m_offset, const int32_t* __restrict__ cu, const int32_t* __restrict__ seq_new, const int32_t* __restrict__ seq_slot,
                        float* __restrict__ kappa, float* __restrict__ tau, float* __restrict__ m_out, float* __restrict__ inv_den, int H, int d,
                        int n_offset) {
    const int head = blockIdx.x, seq = blockIdx.y, lane = threadIdx.x;
    const int count = seq_new[seq];
    if (count <= 0) return;
    const long long row0 = cu[seq];
    float* st = state + (size_t)seq_slot[seq] * state_stride;
    float m = st[m_offset + head];
    float* np = st + (size_t)head * head_stride + n_offset;
    const float b_i = bias[head], b_f = bias[H + head];
    float n[NR], qn[NR], kn[NR];
    const T* qb = q + (size_t)head * d;
    const T* kb = k + (size_t)head * d;
    if (inv_den) {
#pragma unroll
        for (int r = 0; r < NR; ++r) {
            const int i = lane + r * TQK_WAVE;
            n[r] = i < d ? np[i] : 0.f;
            qn[r] = i < d ? to_float(qb[row0 * stride + i]) : 0.f;
            kn[r] = i < d ? to_float(kb[row0 * stride + i]) : 0.f;
        }
    }
    float zi = 0.f, zf = 0.f;
    if (lane < count) { zi = z[(row0 + lane) * z_stride + head]; zf = z[(row0 + lane) * z_stride + H + head]; }
    for (int t0 = 0; t0 < count; t0 += TQK_WAVE) {
        const int nt = min(TQK_WAVE, count - t0);
        const float a = cap * tanhf((zi + b_i) / cap), f = log_sigmoid(cap * tanhf((zf + b_f) / cap));
        if (t0 + TQK_WAVE + lane < count) {
            const long long next = row0 + t0 + TQK_WAVE + lane;
            zi = z[next * z_stride + head];
            zf = z[next * z_stride + H + head];
        }
        float m_mine = 0.f, before = 0.f;
        for (int t = 0; t < nt; ++t) {
            const float m_new = fmaxf(__shfl(f, t, TQK_WAVE) + m, __shfl(a, t, TQK_WAVE));
            if (lane == t) { before = m; m_mine = m_new; }
            m = m_new;
        }
        const float kap = f + before - m_mine, ta = a - m_mine;
        if (lane < nt) {
            const size_t at = (size_t)(row0 + t0 + lane) * H + head;
            kappa[at] = kap;
            tau[at] = ta;
            m_out[at] = m_mine;
        }
        if (!inv_den) continue;
        const float keep_l = expf(kap), take_l = expf(ta), floor_l = expf(-m_mine);
        float mine = 0.f;
        for (int t = 0; t < nt; ++t) {
            float qc[NR], kc[NR];
#pragma unroll
            for (int r = 0; r < NR; ++r) { qc[r] = qn[r]; kc[r] = kn[r]; }
            if (t0 + t + 1 < count) {
                const long long next = row0 + t0 + t + 1;
#pragma unroll
                for (int r = 0; r < NR; ++r) {
                    const int i = lane + r * TQK_WAVE;
                    if (i < d) { qn[r] = to_float(qb[next * stride + i]); kn[r] = to_float(kb[next * stride + i]); }
                }
            }
            const float keep = __shfl(keep_l, t, TQK_WAVE), take = __shfl(take_l, t, TQK_WAVE);
            float dot = 0.f;
#pragma unroll
            for (int r = 0; r < NR; ++r) {
                n[r] = fmaf(keep, n[r], take * kc[r]);
                dot = fmaf(n[r], qc[r] * q_scale, dot);
            }
            dot = wave_sum(dot);
            if (lane == t) mine = 1.f / (fmaxf(fabsf(dot), floor_l) + 1e-6f);
        }
        if (lane < nt) inv_den[(size_t)(row0 + t0 + lane) * H + head] = mine;
    }
    if (lane == 0) st[m_offset + head] = m;
    if (inv_den) {
#pragma unroll
        for (int r = 0; r < NR; ++r) {
            const int i = lane + r * TQK_WAVE;
            if (i < d) np[i] = n[r];
        }
    }
}


// ---- many tokens: the logarithms -----------------------------------------------------------------------
#define ML_SCAN_WAVES 16
__global__ __launch_bounds__(ML_SCAN_WAVES * TQK_WAVE)
void mlstm_gate_scan_kernel(const float* __restrict__ z, long long z_stride, const float* __restrict__ bias, float cap, float* __restrict__ state,
                            long long state_stride, long long m_offset, const int32_t* __restrict__ cu, const int32_t* __restrict__ seq_new,
                            const int32_t* __restrict__ seq_slot, float* __restrict__ kappa, float* __restrict__ tau, float* __restrict__ m_out, int H) {
    __shared__ float sums[2][ML_SCAN_WAVES], tops[2][ML_SCAN_WAVES];
    const int head = blockIdx.x, seq = blockIdx.y;
    const int wave = threadIdx.x / TQK_WAVE, lane = threadIdx.x % TQK_WAVE;
    const int count = seq_new[seq];
    if (count <= 0) return;
    const long long row0 = cu[seq];
    float* mp = state + (size_t)seq_slot[seq] * state_stride + m_offset + head;
    float m = *mp;                                      // every thread carries it
    const float b_i = bias[head], b_f = bias[H + head];
    int turn = 0;
    for (int t0 = 0; t0 < count; t0 += ML_SCAN_WAVES * TQK_WAVE, turn ^= 1) {
        const int t = t0 + threadIdx.x;
        const bool live = t < count;
        float a = -INFINITY, f = 0.f;                   // beyond the last token nothing changes
        if (live) {
            a = cap * tanhf((z[(row0 + t) * z_stride + head] + b_i) / cap);
            f = log_sigmoid(cap * tanhf((z[(row0 + t) * z_stride + H + head] + b_f) / cap));
        }
        float F = f;
#pragma unroll
        for (int o = 1; o < TQK_WAVE; o <<= 1) { const float u = __shfl_up(F, o, TQK_WAVE); if (lane >= o) F += u; }
        float G = live ? a - F : -INFINITY;
#pragma unroll
        for (int o = 1; o < TQK_WAVE; o <<= 1) { const float u = __shfl_up(G, o, TQK_WAVE); if (lane >= o) G = fmaxf(G, u); }
        if (lane == TQK_WAVE - 1) { sums[turn][wave] = F; tops[turn][wave] = G; }
        __syncthreads();                                // (two sets of places in turn: one barrier a round)
        float mine = m;                                 // the maximum in front of this wave's tokens
        for (int w = 0; w < ML_SCAN_WAVES; ++w) {
            if (w == wave) mine = m;
            m = sums[turn][w] + fmaxf(m, tops[turn][w]);
        }
        const float mt = F + fmaxf(mine, G);
        float before = __shfl_up(mt, 1, TQK_WAVE);
        if (lane == 0) before = mine;
        if (live) {
            const size_t at = (size_t)(row0 + t) * H + head;
            kappa[at] = f + before - mt;
            tau[at] = a - mt;
            m_out[at] = mt;
        }
    }
    if (threadIdx.x == 0) *mp = m;
}

// ---- chunks on the matrix cores --------------------------------------------------------------------------
// v_mfma_f32_16x16x32_bf16, D[16x16] += A[16x32] B[32x16]: a lane holds of A row l%16 and of B column l%16 the eight k from 8 (l/16), and of D
// column l%16 the rows 4 (l/16) + i.  Where k runs over tokens, an operand's eight numbers lie in eight rows of memory: a lane then loads four
// neighbouring elements of a row at once, one for each of four tiles, so that row (or column) r of tile j is element 4 r + j of a group of 64.
typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 ml_bf16x8_t;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float ml_floatx4_t;
union ml_pack8 {
    ml_bf16x8_t v;
    uint16_t u[8];
    uint4 q;
};
__device__ __forceinline__ float bits_float(uint32_t b) { return __uint_as_float(b << 16); }
// a float32 number as the sum of two bfloat16 ones
__device__ __forceinline__ void two_parts(float x, uint16_t& hi, uint16_t& lo) {
    hi = float_to_bf16_bits(x);
    lo = float_to_bf16_bits(x - bits_float(hi));
}
// the running sum of kappa over a chunk's tokens, a lane a token (those beyond the chunk add nothing)
__device__ __forceinline__ float running_kappa(const float* __restrict__ kappa, long long row0, int count, int H, int head, int lane) {
    float C = lane < count ? kappa[(row0 + lane) * H + head] : 0.f;
#pragma unroll
    for (int o = 1; o < TQK_WAVE; o <<= 1) { const float u = __shfl_up(C, o, TQK_WAVE); if (lane >= o) C += u; }
    return C;
}

struct MlChunkArgs {
    const bf16_t *q, *k, *v;
    long long stride;
    const float *kappa, *tau, *m;
    const int32_t *chunk_row0, *chunk_count;
    float* chunk_state;             // [chunks][heads][d * dv | d]
    float* chunk_decay;             // [chunks][heads]
    float q_scale;
    float* out;                     // [tokens, heads, dv], or null: then normed and gated rows go to gated
    const float* norm_w;            // [heads][dv]
    float eps;
    const bf16_t* gate;             // rows `stride` apart
    bf16_t* gated;                  // [tokens, heads * dv]
    int H, d, dv, n_chunks;
};

// A wave: 64 key channels by 64 columns of one head of one chunk.
__global__ __launch_bounds__(4 * TQK_WAVE)
void mlstm_local_kernel(const MlChunkArgs a, int n_items) {
    __shared__ float w_lds[4][64];
    const int wave = threadIdx.x / TQK_WAVE, lane = threadIdx.x % TQK_WAVE;
    const int item = blockIdx.x * 4 + wave;
    if (item >= n_items) return;
    const int vts = (a.dv + 63) / 64, dts = (a.d + 63) / 64;
    const int v0 = (item % vts) * 64, d0 = (item / vts % dts) * 64, head = item / (vts * dts) % a.H, chunk = item / (vts * dts * a.H);
    const int g = lane / 16, r = lane % 16;
    const long long row0 = a.chunk_row0[chunk];
    const int count = a.chunk_count[chunk];
    const float C = running_kappa(a.kappa, row0, count, a.H, head, lane);
    const float end = __shfl(C, TQK_WAVE - 1, TQK_WAVE);
    w_lds[wave][lane] = lane < count ? expf(end - C + a.tau[(row0 + lane) * a.H + head]) : 0.f;
    // (written and read by the same wave: what waits for the reads is the compiler's own wait)
    const bool d_in = d0 + 4 * r < a.d, v_in = v0 + 4 * r < a.dv;
    const bf16_t* kb = a.k + (size_t)head * a.d + (d_in ? d0 + 4 * r : 0);
    const bf16_t* vb = a.v + (size_t)head * a.dv + (v_in ? v0 + 4 * r : 0);
    uint2 kr[2][8], vr[2][8];
#pragma unroll
    for (int ks = 0; ks < 2; ++ks)
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const long long row = row0 + min(32 * ks + 8 * g + e, count - 1);
            kr[ks][e] = *reinterpret_cast<const uint2*>(kb + row * a.stride);
            vr[ks][e] = *reinterpret_cast<const uint2*>(vb + row * a.stride);
        }
    __builtin_amdgcn_wave_barrier();
    ml_floatx4_t acc[4][4];
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int c = 0; c < 4; ++c) acc[j][c] = ml_floatx4_t{0.f, 0.f, 0.f, 0.f};
    float n4[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
        ml_pack8 hi[4], lo[4], vv[4];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const float w = d_in ? w_lds[wave][32 * ks + 8 * g + e] : 0.f;
            const uint2 kk = kr[ks][e];
            const float k4[4] = {bits_float(kk.x & 0xffff), bits_float(kk.x >> 16), bits_float(kk.y & 0xffff), bits_float(kk.y >> 16)};
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const float x = k4[j] * w;
                n4[j] += x;
                two_parts(x, hi[j].u[e], lo[j].u[e]);
            }
            const uint2 vq = vr[ks][e];
            vv[0].u[e] = (uint16_t)vq.x; vv[1].u[e] = (uint16_t)(vq.x >> 16);
            vv[2].u[e] = (uint16_t)vq.y; vv[3].u[e] = (uint16_t)(vq.y >> 16);
        }
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
            for (int c = 0; c < 4; ++c) {
                acc[j][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi[j].v, vv[c].v, acc[j][c], 0, 0, 0);
                acc[j][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo[j].v, vv[c].v, acc[j][c], 0, 0, 0);
            }
    }
    const size_t per_head = (size_t)a.d * a.dv + a.d;
    float* S = a.chunk_state + ((size_t)chunk * a.H + head) * per_head;
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int ch = d0 + 4 * (4 * g + i) + j;
            if (ch < a.d && v_in)
                *reinterpret_cast<float4*>(S + (size_t)ch * a.dv + v0 + 4 * r) = make_float4(acc[j][0][i], acc[j][1][i], acc[j][2][i], acc[j][3][i]);
        }
    if (v0 == 0) {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            n4[j] += __shfl_xor(n4[j], 16, TQK_WAVE);
            n4[j] += __shfl_xor(n4[j], 32, TQK_WAVE);
        }
        if (g == 0 && d_in) *reinterpret_cast<float4*>(S + (size_t)a.d * a.dv + d0 + 4 * r) = make_float4(n4[0], n4[1], n4[2], n4[3]);
        if (d0 == 0 && lane == 0) a.chunk_decay[(size_t)chunk * a.H + head] = expf(end);
    }
}

// A block of four waves: one head of one chunk and up to NG groups of 64 columns.  First a wave works out P for 16 of the chunk's tokens (and
// their denominators) and leaves it in LDS; then it takes a group of columns for NG of the four sets of 16 tokens.
#define ML_PROW 72                  // numbers between rows of P in LDS (16 bytes more than a row, against bank conflicts)
template <int NG>
__global__ __launch_bounds__(4 * TQK_WAVE)
void mlstm_apply_kernel(const MlChunkArgs a) {
    __shared__ __attribute__((aligned(16))) uint16_t p_hi[64 * ML_PROW], p_lo[64 * ML_PROW];
    __shared__ float c_lds[64], u_lds[64], inter[64], inv_den[64], ss_lds[NG][64];
    const int wave = threadIdx.x / TQK_WAVE, lane = threadIdx.x % TQK_WAVE;
    const int g = lane / 16, r = lane % 16;
    const int head = blockIdx.y, chunk = blockIdx.z;
    const long long row0 = a.chunk_row0[chunk];
    const int count = a.chunk_count[chunk];
    const int d = a.d, dv = a.dv, H = a.H;
    const size_t per_head = (size_t)d * dv + d;
    const float* S = a.chunk_state + ((size_t)chunk * H + head) * per_head;
    const float* n0 = S + (size_t)d * dv;
    const bf16_t* qb = a.q + (size_t)head * d;
    const bf16_t* kb = a.k + (size_t)head * d;
    if (wave == 0) {
        const float C = running_kappa(a.kappa, row0, count, H, head, lane);
        c_lds[lane] = C;
        u_lds[lane] = lane < count ? a.tau[(row0 + lane) * H + head] - C : -INFINITY;
    }
    __syncthreads();
    const int kbs = (d + 31) / 32;
    {
        const int t = 16 * wave + r;
        const bf16_t* qr = qb + (row0 + min(t, count - 1)) * a.stride;
        ml_floatx4_t s[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) s[j] = ml_floatx4_t{0.f, 0.f, 0.f, 0.f};
        float qn = 0.f;
        for (int kk = 0; kk < kbs; ++kk) {
            const int e0 = 32 * kk + 8 * g;
            const bool in = e0 < d;                     // (d is a multiple of 8: a piece is inside or outside)
            const int e0c = in ? e0 : 0;
            ml_pack8 bq, ak[4];
            bq.q = *reinterpret_cast<const uint4*>(qr + e0c);
#pragma unroll
            for (int j = 0; j < 4; ++j) ak[j].q = *reinterpret_cast<const uint4*>(kb + (row0 + min(16 * j + r, count - 1)) * a.stride + e0c);
            const float4 n_a = *reinterpret_cast<const float4*>(n0 + e0c), n_b = *reinterpret_cast<const float4*>(n0 + e0c + 4);
            if (!in) bq.q = make_uint4(0, 0, 0, 0);
            const float n8[8] = {n_a.x, n_a.y, n_a.z, n_a.w, n_b.x, n_b.y, n_b.z, n_b.w};
#pragma unroll
            for (int e = 0; e < 8; ++e) qn = fmaf(bits_float(bq.u[e]), n8[e], qn);
#pragma unroll
            for (int j = 0; j < 4; ++j)
                if (j <= wave) s[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ak[j].v, bq.v, s[j], 0, 0, 0);
        }
        const float Ct = c_lds[t];
        float sum = 0.f;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            if (j > (wave | 1)) continue;               // (the other of two sets of 16 keys that are read together holds zeros)
            uint16_t h4[4], l4[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int key = 16 * j + 4 * g + i;
                const float p = key <= t && j <= wave ? s[j][i] * a.q_scale * expf(Ct + u_lds[key]) : 0.f;
                sum += p;
                two_parts(p, h4[i], l4[i]);
            }
            const int at = t * ML_PROW + 16 * j + 4 * g;
            *reinterpret_cast<uint2*>(p_hi + at) = make_uint2(h4[0] | ((uint32_t)h4[1] << 16), h4[2] | ((uint32_t)h4[3] << 16));
            *reinterpret_cast<uint2*>(p_lo + at) = make_uint2(l4[0] | ((uint32_t)l4[1] << 16), l4[2] | ((uint32_t)l4[3] << 16));
        }
        sum += __shfl_xor(sum, 16, TQK_WAVE);
        sum += __shfl_xor(sum, 32, TQK_WAVE);
        qn += __shfl_xor(qn, 16, TQK_WAVE);
        qn += __shfl_xor(qn, 32, TQK_WAVE);
        if (g == 0) {
            const float from_state = expf(Ct) * a.q_scale;
            inter[t] = from_state;
            const float floor_t = t < count ? expf(-a.m[(row0 + t) * H + head]) : 1.f;
            inv_den[t] = 1.f / (fmaxf(fabsf(fmaf(from_state, qn, sum)), floor_t) + 1e-6f);
        }
    }
    __syncthreads();
    const int group = wave % NG, first = wave / NG * NG;       // the wave's columns and its first set of 16 tokens
    const int v0 = blockIdx.x * 64 * NG + 64 * group;
    const bool v_in = v0 + 4 * r < dv;
    const bool works = v0 < dv && 16 * first < count;
    ml_floatx4_t acc[NG][4];
#pragma unroll
    for (int tt = 0; tt < NG; ++tt)
#pragma unroll
        for (int c = 0; c < 4; ++c) acc[tt][c] = ml_floatx4_t{0.f, 0.f, 0.f, 0.f};
    if (works) {
        // what lies in the state the chunk starts from
        const float* Sc = S + (v_in ? v0 + 4 * r : 0);
        for (int kk = 0; kk < kbs; ++kk) {
            const int e0 = 32 * kk + 8 * g;
            const bool in = e0 < d;
            const int e0c = in ? e0 : 0;
            float4 s8[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) s8[e] = *reinterpret_cast<const float4*>(Sc + (size_t)(e0c + e) * dv);
            ml_pack8 aq[NG], hi[4], lo[4];
#pragma unroll
            for (int tt = 0; tt < NG; ++tt) {
                aq[tt].q = *reinterpret_cast<const uint4*>(qb + (row0 + min(16 * (first + tt) + r, count - 1)) * a.stride + e0c);
                if (!in) aq[tt].q = make_uint4(0, 0, 0, 0);
            }
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                two_parts(s8[e].x, hi[0].u[e], lo[0].u[e]);
                two_parts(s8[e].y, hi[1].u[e], lo[1].u[e]);
                two_parts(s8[e].z, hi[2].u[e], lo[2].u[e]);
                two_parts(s8[e].w, hi[3].u[e], lo[3].u[e]);
            }
#pragma unroll
            for (int tt = 0; tt < NG; ++tt)
#pragma unroll
                for (int c = 0; c < 4; ++c) {
                    acc[tt][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(aq[tt].v, hi[c].v, acc[tt][c], 0, 0, 0);
                    acc[tt][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(aq[tt].v, lo[c].v, acc[tt][c], 0, 0, 0);
                }
        }
#pragma unroll
        for (int tt = 0; tt < NG; ++tt)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const float f = inter[16 * (first + tt) + 4 * g + i];
#pragma unroll
                for (int c = 0; c < 4; ++c) acc[tt][c][i] *= f;
            }
        // what the chunk's own tokens give
        const bf16_t* vb = a.v + (size_t)head * dv + (v_in ? v0 + 4 * r : 0);
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
            if (32 * ks >= 16 * (first + NG) || 32 * ks >= count) continue;        // tokens behind every one of the wave's
            uint2 vr[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) vr[e] = *reinterpret_cast<const uint2*>(vb + (row0 + min(32 * ks + 8 * g + e, count - 1)) * a.stride);
            ml_pack8 vv[4];
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                vv[0].u[e] = (uint16_t)vr[e].x; vv[1].u[e] = (uint16_t)(vr[e].x >> 16);
                vv[2].u[e] = (uint16_t)vr[e].y; vv[3].u[e] = (uint16_t)(vr[e].y >> 16);
            }
#pragma unroll
            for (int tt = 0; tt < NG; ++tt) {
                if (16 * (first + tt) + 15 < 32 * ks) continue;                     // (nothing of P was written there)
                ml_pack8 ph, pl;
                const int at = (16 * (first + tt) + r) * ML_PROW + 32 * ks + 8 * g;
                ph.q = *reinterpret_cast<const uint4*>(p_hi + at);
                pl.q = *reinterpret_cast<const uint4*>(p_lo + at);
#pragma unroll
                for (int c = 0; c < 4; ++c) {
                    acc[tt][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ph.v, vv[c].v, acc[tt][c], 0, 0, 0);
                    acc[tt][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pl.v, vv[c].v, acc[tt][c], 0, 0, 0);
                }
            }
        }
#pragma unroll
        for (int tt = 0; tt < NG; ++tt)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int t = 16 * (first + tt) + 4 * g + i;
                const float f = v_in ? inv_den[t] : 0.f;
#pragma unroll
                for (int c = 0; c < 4; ++c) acc[tt][c][i] *= f;
                if (a.out && v_in && t < count)
                    *reinterpret_cast<float4*>(a.out + ((size_t)(row0 + t) * H + head) * dv + v0 + 4 * r) =
                        make_float4(acc[tt][0][i], acc[tt][1][i], acc[tt][2][i], acc[tt][3][i]);
            }
    }
    if (a.out) return;
    // the head's norm, the weight and the gate: the sums of squares of the groups of columns meet in LDS
#pragma unroll
    for (int tt = 0; tt < NG; ++tt)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            float ss = 0.f;
#pragma unroll
            for (int c = 0; c < 4; ++c) ss = fmaf(acc[tt][c][i], acc[tt][c][i], ss);
#pragma unroll
            for (int o = 1; o < 16; o <<= 1) ss += __shfl_xor(ss, o, TQK_WAVE);
            if (r == 0) ss_lds[group][16 * (first + tt) + 4 * g + i] = ss;
        }
    __syncthreads();
    if (!works || !v_in) return;
    const float4 w4 = *reinterpret_cast<const float4*>(a.norm_w + (size_t)head * dv + v0 + 4 * r);
#pragma unroll
    for (int tt = 0; tt < NG; ++tt)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = 16 * (first + tt) + 4 * g + i;
            if (t >= count) continue;
            float ss = 0.f;
#pragma unroll
            for (int w = 0; w < NG; ++w) ss += ss_lds[w][t];
            const float inv = 1.f / sqrtf(ss / (float)dv + a.eps);
            const uint2 gq = *reinterpret_cast<const uint2*>(a.gate + (row0 + t) * a.stride + (size_t)head * dv + v0 + 4 * r);
            const float g4[4] = {bits_float(gq.x & 0xffff), bits_float(gq.x >> 16), bits_float(gq.y & 0xffff), bits_float(gq.y >> 16)};
            const float ww[4] = {w4.x, w4.y, w4.z, w4.w};
            uint16_t o4[4];
#pragma unroll
            for (int c = 0; c < 4; ++c) o4[c] = float_to_bf16_bits(acc[tt][c][i] * inv * ww[c] / (1.f + expf(-g4[c])));
            *reinterpret_cast<uint2*>(a.gated + ((size_t)(row0 + t) * H + head) * dv + v0 + 4 * r) =
                make_uint2(o4[0] | ((uint32_t)o4[1] << 16), o4[2] | ((uint32_t)o4[3] << 16));
        }
}

extern "C" int tqk_mlstm_gate_scan(const float* z, long long z_stride, const float* bias, float cap, float* state, long long state_stride, long long m_offset,
                                   const int32_t* cu, const int32_t* seq_new, const int32_t* seq_slot, float* kappa, float* tau, float* m, int n_seqs,
                                   int heads, void* stream) {
    TQK_REQUIRE(z && bias && state && cu && seq_new && seq_slot && kappa && tau && m, "tqk_mlstm_gate_scan: null pointer");
    TQK_REQUIRE(n_seqs >= 0 && n_seqs <= 65535 && heads > 0 && z_stride >= 2 * heads && cap > 0.f && state_stride >= m_offset + heads,
                "tqk_mlstm_gate_scan: bad sizes");
    if (n_seqs == 0) return 0;
    mlstm_gate_scan_kernel<<<dim3(heads, n_seqs), ML_SCAN_WAVES * TQK_WAVE, 0, (hipStream_t)stream>>>(z, z_stride, bias, cap, state, state_stride, m_offset, cu,
                                                                                                       seq_new, seq_slot, kappa, tau, m, heads);
    return tqk_check_launch("tqk_mlstm_gate_scan");
}

extern "C" int tqk_mlstm_chunks_supported(int d, int dv) { return d > 0 && d % 8 == 0 && d <= ML_MAX_D && dv > 0 && dv % 4 == 0 && dv <= 65535; }
extern "C" int tqk_mlstm_apply_norms(int dv) { return dv <= 256; }

static int mlstm_chunk_args(MlChunkArgs& a, const void* q, const void* k, const void* v, long long stride, const float* kappa, const float* tau,
                            const int32_t* chunk_row0, const int32_t* chunk_count, int n_chunks, float* chunk_state, int heads, int d, int dv) {
    TQK_REQUIRE(q && k && v && kappa && tau && chunk_row0 && chunk_count && chunk_state, "tqk_mlstm chunks: null pointer");
    TQK_REQUIRE(tqk_mlstm_chunks_supported(d, dv), "tqk_mlstm chunks: heads of %d and %d elements are not taken", d, dv);
    TQK_REQUIRE(n_chunks >= 0 && n_chunks <= 65535 && heads > 0 && heads <= 65535, "tqk_mlstm chunks: bad sizes");
    TQK_REQUIRE(stride % 8 == 0 && ((((uintptr_t)q | (uintptr_t)k | (uintptr_t)chunk_state) & 15) | ((uintptr_t)v & 7)) == 0,
                "tqk_mlstm chunks: rows of q and k must begin at multiples of 16 bytes, of v at multiples of 8");
    a = {};
    a.q = (const bf16_t*)q; a.k = (const bf16_t*)k; a.v = (const bf16_t*)v; a.stride = stride;
    a.kappa = kappa; a.tau = tau; a.chunk_row0 = chunk_row0; a.chunk_count = chunk_count; a.chunk_state = chunk_state;
    a.H = heads; a.d = d; a.dv = dv; a.n_chunks = n_chunks;
    return 0;
}

extern "C" int tqk_mlstm_local(const void* k, const void* v, long long stride, const float* kappa, const float* tau, const int32_t* chunk_row0,
                               const int32_t* chunk_count, int n_chunks, float* chunk_state, float* chunk_decay, int heads, int d, int dv, void* stream) {
    MlChunkArgs a;
    if (mlstm_chunk_args(a, k, k, v, stride, kappa, tau, chunk_row0, chunk_count, n_chunks, chunk_state, heads, d, dv)) return -1;
    TQK_REQUIRE(chunk_decay, "tqk_mlstm_local: null pointer");
    a.chunk_decay = chunk_decay;
    const long long items = (long long)n_chunks * heads * ((d + 63) / 64) * ((dv + 63) / 64);
    TQK_REQUIRE(items <= 0x7fffffff, "tqk_mlstm_local: too many chunks");
    if (items == 0) return 0;
    mlstm_local_kernel<<<(unsigned)((items + 3) / 4), 4 * TQK_WAVE, 0, (hipStream_t)stream>>>(a, (int)items);
    return tqk_check_launch("tqk_mlstm_local");
}

extern "C" int tqk_mlstm_apply(const void* q, const void* k, const void* v, long long stride, const float* kappa, const float* tau, const float* m,
                               float q_scale, const int32_t* chunk_row0, const int32_t* chunk_count, int n_chunks, float* chunk_state, float* out,
                               const float* norm_weight, float eps, const void* gate, void* gated, int heads, int d, int dv, void* stream) {
    MlChunkArgs a;
    if (mlstm_chunk_args(a, q, k, v, stride, kappa, tau, chunk_row0, chunk_count, n_chunks, chunk_state, heads, d, dv)) return -1;
    TQK_REQUIRE(m, "tqk_mlstm_apply: null pointer");
    TQK_REQUIRE(out || (norm_weight && gate && gated && tqk_mlstm_apply_norms(dv)), "tqk_mlstm_apply: nowhere to write to, or heads too large to norm here");
    TQK_REQUIRE((((uintptr_t)out | (uintptr_t)norm_weight) & 15) == 0 && (((uintptr_t)gate | (uintptr_t)gated) & 7) == 0, "tqk_mlstm_apply: operands are not aligned");
    if (n_chunks == 0) return 0;
    a.m = m; a.q_scale = q_scale; a.out = out; a.norm_w = norm_weight; a.eps = eps; a.gate = (const bf16_t*)gate; a.gated = (bf16_t*)gated;
    hipStream_t s = (hipStream_t)stream;
    const int ng = dv <= 64 ? 1 : dv <= 128 ? 2 : 4;
    dim3 grid((dv + 64 * ng - 1) / (64 * ng), heads, n_chunks);
    if (ng == 1) mlstm_apply_kernel<1><<<grid, 4 * TQK_WAVE, 0, s>>>(a);
    else if (ng == 2) mlstm_apply_kernel<2><<<grid, 4 * TQK_WAVE, 0, s>>>(a);
    else mlstm_apply_kernel<4><<<grid, 4 * TQK_WAVE, 0, s>>>(a);
    return tqk_check_launch("tqk_mlstm_apply");
}

extern "C" int tqk_mlstm_gates(const float* z, long long z_stride, const float* bias, float cap, const void* q, const void* k, int act_dtype, long long stride,
                               float q_scale, float* state, long long state_stride, long long head_stride, long long m_offset, const int32_t* cu,
                               const int32_t* seq_new, const int32_t* seq_slot, float* kappa, float* tau, float* m, float* inv_den, int n_seqs, int heads,
                               int d, void* stream) {
    TQK_REQUIRE(z && bias && state && cu && seq_new && seq_slot && kappa && tau && m, "tqk_mlstm_gates: null pointer");
    TQK_REQUIRE(!inv_den || (q && k), "tqk_mlstm_gates: the denominators need q and k");
    TQK_REQUIRE(n_seqs >= 0 && n_seqs <= 65535 && heads > 0 && d > 0 && d <= ML_MAX_D && z_stride >= 2 * heads, "tqk_mlstm_gates: bad sizes");
    TQK_REQUIRE(cap > 0.f, "tqk_mlstm_gates: the gates' cap must be positive");
    TQK_REQUIRE(head_stride >= d && m_offset >= head_stride * heads && state_stride >= m_offset + heads, "tqk_mlstm_gates: the state's parts overlap");
    if (n_seqs == 0) return 0;
    const int n_offset = (int)(head_stride - d);
    hipStream_t s = (hipStream_t)stream;
    dim3 grid(heads, n_seqs);
#define TQK_MLG(T, NR) mlstm_gates_kernel<T, NR><<<grid, TQK_WAVE, 0, s>>>(z, z_stride, bias, cap, (const T*)q, (const T*)k, stride, q_scale, state, state_stride, \
        head_stride, m_offset, cu, seq_new, seq_slot, kappa, tau, m, inv_den, heads, d, n_offset)
#define TQK_MLG_D(T) do { if (d <= 64) TQK_MLG(T, 1); else if (d <= 128) TQK_MLG(T, 2); else if (d <= 256) TQK_MLG(T, 4); else TQK_MLG(T, 8); } while (0)
    if (act_dtype == TQK_F32) TQK_MLG_D(float);
    else if (act_dtype == TQK_BF16) TQK_MLG_D(bf16_t);
    else return tqk_fail("tqk_mlstm_gates: unknown dtype %d", act_dtype);
#undef TQK_MLG_D
#undef TQK_MLG
    return tqk_check_launch("tqk_mlstm_gates");
}
