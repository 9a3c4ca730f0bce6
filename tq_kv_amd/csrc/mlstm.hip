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
