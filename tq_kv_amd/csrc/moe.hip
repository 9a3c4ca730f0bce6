// A feed-forward of routed experts: the router, the grouping of a step's (token, expert) pairs by
// expert, the experts' products over the grouped rows, and the weighted sum.
//
//   route     z = W_r x in float32, s = softmax(z) over all experts, the `top` largest (the lower index wins
//             a tie); weight = s * scale, not renormalised.  One wave per token.  Mode bit 1 renormalises over the chosen;
//             mode bit 2 makes every expert's score sigmoid(z) on its own instead of the softmax.
//   route_grouped   the same logits over experts and, after them, experts that give back their input; chosen by s + correction within
//             the best groups of neighbours (a group's rank is its largest s + correction), weights the chosen s over (their sum + floor)
//   scale     rows[pair_pos[p]] = weight[p] * x[p / top] (for experts whose input, not output, carries the weight), and unit[p] = 1
//   group     pair p = (token p / top, choice p % top) gets a row of its own among its expert's rows:
//             pair_pos[p]; sorted_tok[row] names the row's token.  The rows of an expert are cut into tiles of
//             tile_m rows; the tile list (expert, first row, rows) and its length stay on the device, so the
//             launches that follow have the same shape whatever the router chose.  A choice beyond the experts with weights
//             (an expert that gives back its input) gets no row: pair_pos[p] = -1.
//   product   for each tile, rows x (gathered through sorted_tok, or as they lie) times the tile's expert's
//             weight: plain, or gate and up with the gate applied.  Blocks beyond the list's length exit.
//   combine   out[t] = sum_k weight[t, k] * y[pair_pos[t, k]] (+ what a shared expert gave), in float32; the token's own input in
//             place of a row where there is none; optionally out[t] = scale (that + beside[t]).
//
// A row's sums never depend on which rows share its tile, nor on the order the pairs were given rows in.
#include "common.h"
#include "tq_kernels.h"

#define MOE_MAX_EXPERTS 512
#define MOE_ROUTE_WAVES 16
#define MOE_ROUTE_TOKENS 4     // tokens of a block in steps of many
#define MOE_TM 32               // rows of a tile
#define MOE_TN 64               // features of a block
#define MOE_TK 16               // k per stage

// ---- route -----------------------------------------------------------------------------------
// A block takes NT tokens: its waves share the experts out for the logits, two at once (dot products over the lanes, several loads under way
// together, added up in an order that the row's length alone decides), then a wave per token takes the softmax and the largest.
// Logit e of the block's token n goes to z[n * MOE_MAX_EXPERTS + e].  One row more where a gate is given: sigmoid(x . gate_w) per token, which
// rides along with the experts' dot products.
template <typename TA, typename TW, int NT>
__device__ __forceinline__ void route_logits(const TA* __restrict__ x, int n_tokens, const TW* __restrict__ w, int n_experts, int hidden,
                                             const TW* __restrict__ gate_w, float* __restrict__ gate_out, float* z) {
    const int wave = threadIdx.x / TQK_WAVE, lane = threadIdx.x % TQK_WAVE;
    const int t0 = blockIdx.x * NT, rows = n_experts + (gate_w ? 1 : 0);
    const TA* xr[NT];
#pragma unroll
    for (int n = 0; n < NT; ++n) xr[n] = x + (size_t)min(t0 + n, n_tokens - 1) * hidden;
    for (int e0 = wave; e0 < rows; e0 += 2 * MOE_ROUTE_WAVES) {
        const int ee[2] = {e0, min(e0 + MOE_ROUTE_WAVES, rows - 1)};
        const TW* wr[2];
#pragma unroll
        for (int j = 0; j < 2; ++j) wr[j] = ee[j] < n_experts ? w + (size_t)ee[j] * hidden : gate_w;
        float d[2][NT][4];
#pragma unroll
        for (int j = 0; j < 2; ++j)
#pragma unroll
            for (int n = 0; n < NT; ++n) d[j][n][0] = d[j][n][1] = d[j][n][2] = d[j][n][3] = 0.f;
        if (sizeof(TA) == 2 && sizeof(TW) == 2 && hidden % 8 == 0) {
            // bfloat16 rows whose length is a multiple of 8: 16 bytes a lane and load
#pragma unroll 2
            for (int c = lane * 8; c < hidden; c += TQK_WAVE * 8) {
                uint4 wv[2], xv[NT];
#pragma unroll
                for (int j = 0; j < 2; ++j) wv[j] = *reinterpret_cast<const uint4*>(wr[j] + c);
#pragma unroll
                for (int n = 0; n < NT; ++n) xv[n] = *reinterpret_cast<const uint4*>(xr[n] + c);
#pragma unroll
                for (int j = 0; j < 2; ++j)
#pragma unroll
                    for (int n = 0; n < NT; ++n) {
                        const uint32_t xw[4] = {xv[n].x, xv[n].y, xv[n].z, xv[n].w}, ww[4] = {wv[j].x, wv[j].y, wv[j].z, wv[j].w};
#pragma unroll
                        for (int k = 0; k < 4; ++k) {
                            d[j][n][k] = fmaf(__uint_as_float(xw[k] << 16), __uint_as_float(ww[k] << 16), d[j][n][k]);
                            d[j][n][k] = fmaf(__uint_as_float(xw[k] & 0xffff0000u), __uint_as_float(ww[k] & 0xffff0000u), d[j][n][k]);
                        }
                    }
            }
        } else {
            for (int c = lane; c < hidden; c += 4 * TQK_WAVE) {
#pragma unroll
                for (int k = 0; k < 4; ++k) {
                    const int i = c + k * TQK_WAVE;
                    if (i >= hidden) continue;
#pragma unroll
                    for (int j = 0; j < 2; ++j)
#pragma unroll
                        for (int n = 0; n < NT; ++n) d[j][n][k] = fmaf(to_float(xr[n][i]), to_float(wr[j][i]), d[j][n][k]);
                }
            }
        }
#pragma unroll
        for (int j = 0; j < 2; ++j)
#pragma unroll
            for (int n = 0; n < NT; ++n) {
                const float dot = wave_sum((d[j][n][0] + d[j][n][1]) + (d[j][n][2] + d[j][n][3]));
                if (lane != 0 || e0 + j * MOE_ROUTE_WAVES >= rows || t0 + n >= n_tokens) continue;
                if (ee[j] < n_experts) z[n * MOE_MAX_EXPERTS + ee[j]] = dot;
                else gate_out[t0 + n] = 1.f / (1.f + expf(-dot));
            }
    }
    __syncthreads();
}

template <typename TA, typename TW, int NT>
__global__ __launch_bounds__(MOE_ROUTE_WAVES * TQK_WAVE)
void moe_route_kernel(const TA* __restrict__ x, int n_tokens, const TW* __restrict__ w, int n_experts, int hidden, int top, float scale, int mode,
                      int32_t* __restrict__ idx, float* __restrict__ weight, const TW* __restrict__ gate_w, float* __restrict__ gate_out) {
    const int renormalize = mode & 1, sigmoid_scores = mode & 2;
    __shared__ float logits[NT * MOE_MAX_EXPERTS];
    const int wave = threadIdx.x / TQK_WAVE, lane = threadIdx.x % TQK_WAVE;
    route_logits<TA, TW, NT>(x, n_tokens, w, n_experts, hidden, gate_w, gate_out, logits);
    const int t = blockIdx.x * NT + wave;
    if (wave >= NT || t >= n_tokens) return;
    float* z = logits + wave * MOE_MAX_EXPERTS;
    float m = -INFINITY;
    for (int e = lane; e < n_experts; e += TQK_WAVE) m = fmaxf(m, z[e]);
    m = wave_max(m);
    float sum = 0.f;
    for (int e = lane; e < n_experts; e += TQK_WAVE) sum += expf(z[e] - m);
    sum = wave_sum(sum);
    // what the lane's experts still offer; a chosen one is struck out in the registers of the lane that holds it
    for (int k = 0; k < top; ++k) {
        float best = -INFINITY;
        int best_e = 0x7fffffff;
        for (int e = lane; e < n_experts; e += TQK_WAVE) {
            const float v = z[e];
            if (v > best) { best = v; best_e = e; }         // increasing e: the lower index stays on a tie
        }
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) {
            const float ov = __shfl_xor(best, o, TQK_WAVE);
            const int oe = __shfl_xor(best_e, o, TQK_WAVE);
            if (ov > best || (ov == best && oe < best_e)) { best = ov; best_e = oe; }
        }
        if (best_e >= n_experts) best_e = k;                        // (scores that are not numbers: some expert that is there)
        if (lane == best_e % TQK_WAVE) z[best_e] = -INFINITY;       // the lane that reads this expert writes it: no other sees it
        if (lane == 0) {
            idx[(size_t)t * top + k] = best_e;
            weight[(size_t)t * top + k] = (sigmoid_scores ? 1.f / (1.f + expf(-best)) : expf(best - m) / sum) * scale;
        }
    }
    if (!renormalize) return;
    // the softmax over the chosen logits alone: the chosen scores divided by their sum, added up in the order they were chosen
    if (lane == 0) {
        float chosen = 0.f;
        for (int k = 0; k < top; ++k) chosen += weight[(size_t)t * top + k];
        for (int k = 0; k < top; ++k) weight[(size_t)t * top + k] /= chosen;
    }
}

// The wave's largest value, by moves between the lanes' registers (inside rows of 16 lanes, then from row to row): no trip through LDS.
template <int CTRL, int ROWS> __device__ __forceinline__ float lanes_max(float v) {
    return fmaxf(v, __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(__builtin_bit_cast(int, -INFINITY), __builtin_bit_cast(int, v), CTRL, ROWS, 0xf, false)));
}
__device__ __forceinline__ float lanes_wave_max(float v) {
    v = lanes_max<0x111, 0xf>(v);           // from the lane 1, 2, 4, 8 places before
    v = lanes_max<0x112, 0xf>(v);
    v = lanes_max<0x114, 0xf>(v);
    v = lanes_max<0x118, 0xf>(v);
    v = lanes_max<0x142, 0xa>(v);           // a row's last lane to the row behind it, then the second row's to the upper two
    v = lanes_max<0x143, 0xc>(v);
    return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), TQK_WAVE - 1));
}
// The lane's largest of z[lane], z[lane + 64], ... below n, then the wave's: the lower index wins a tie.  In every lane of the wave.
__device__ __forceinline__ int wave_argmax(const volatile float* z, int n, int lane, float& best) {
    int at = 0x7fffffff;
    float mine = -INFINITY;
    for (int e = lane; e < n; e += TQK_WAVE) {
        const float v = z[e];
        if (v > mine) { mine = v; at = e; }
    }
    best = lanes_wave_max(mine);
    uint64_t who = __ballot(mine == best && at != 0x7fffffff);
    int first = 0x7fffffff;
    while (who) {                           // (one lane, but for equal values)
        const int l = __builtin_ctzll(who);
        first = min(first, __builtin_amdgcn_readlane(at, l));
        who &= who - 1;
    }
    return first;
}

// Choice by score plus correction within the best groups of neighbours, by a token's wave.  What it keeps of the experts lies in LDS (z: the logits,
// then the scores; choice; group) and is read and written by that wave alone, each element by one lane between two of the wave's exchanges.
__device__ __forceinline__ void choose_grouped(volatile float* z, volatile float* choice, volatile float* group, int n_experts, int top,
                                               const float* __restrict__ correction, int n_groups, int keep, float floor, int lane, int32_t* __restrict__ idx,
                                               float* __restrict__ weight) {
    float m = -INFINITY;
    for (int e = lane; e < n_experts; e += TQK_WAVE) m = fmaxf(m, z[e]);
    m = wave_max(m);
    float sum = 0.f;
    for (int e = lane; e < n_experts; e += TQK_WAVE) sum += expf(z[e] - m);
    sum = wave_sum(sum);
    for (int e = lane; e < n_experts; e += TQK_WAVE) {
        const float s = expf(z[e] - m) / sum;
        z[e] = s;
        choice[e] = s + (correction ? correction[e] : 0.f);
    }
    __threadfence_block();
    __builtin_amdgcn_wave_barrier();
    float best;
    if (keep < n_groups) {
        const int per = n_experts / n_groups;
        for (int g = lane; g < n_groups; g += TQK_WAVE) {
            float b = -INFINITY;
            for (int i = 0; i < per; ++i) b = fmaxf(b, choice[g * per + i]);
            group[g] = b;
        }
        __threadfence_block();
        __builtin_amdgcn_wave_barrier();
        // the kept groups are struck from the list; what is left on it is then closed
        for (int k = 0; k < keep; ++k) {
            const int g = wave_argmax(group, n_groups, lane, best);
            if (g < n_groups && lane == g % TQK_WAVE) group[g] = -INFINITY;
        }
        __threadfence_block();
        __builtin_amdgcn_wave_barrier();
        for (int e = lane; e < n_experts; e += TQK_WAVE)
            if (group[e / per] != -INFINITY) choice[e] = -INFINITY;
        __threadfence_block();
        __builtin_amdgcn_wave_barrier();
    }
    float chosen = 0.f;
    for (int k = 0; k < top; ++k) {
        int e = wave_argmax(choice, n_experts, lane, best);
        e = e < n_experts ? e : k;                          // (scores that are not numbers: some expert that is there)
        if (lane == e % TQK_WAVE) choice[e] = -INFINITY;
        const float s = z[e];
        chosen += s;
        if (lane == 0) {
            idx[k] = e;
            weight[k] = s;
        }
    }
    if (lane == 0)
        for (int k = 0; k < top; ++k) weight[k] /= chosen + floor;
}

template <typename TA, typename TW, int NT>
__global__ __launch_bounds__(MOE_ROUTE_WAVES * TQK_WAVE)
void moe_route_grouped_kernel(const TA* __restrict__ x, int n_tokens, const TW* __restrict__ w, int n_experts, int hidden, int top, const float* __restrict__ correction,
                              int n_groups, int keep, float floor, int32_t* __restrict__ idx, float* __restrict__ weight) {
    __shared__ float logits[NT * MOE_MAX_EXPERTS];
    __shared__ volatile float choices[NT * MOE_MAX_EXPERTS], groups[NT * MOE_MAX_EXPERTS];
    const int wave = threadIdx.x / TQK_WAVE, lane = threadIdx.x % TQK_WAVE;
    route_logits<TA, TW, NT>(x, n_tokens, w, n_experts, hidden, (const TW*)nullptr, (float*)nullptr, logits);
    const int t = blockIdx.x * NT + wave;
    if (wave >= NT || t >= n_tokens) return;
    choose_grouped(logits + wave * MOE_MAX_EXPERTS, choices + wave * MOE_MAX_EXPERTS, groups + wave * MOE_MAX_EXPERTS, n_experts, top, correction, n_groups, keep, floor,
                   lane, idx + (size_t)t * top, weight + (size_t)t * top);
}

// the same from logits that a product has left, [tokens, n_experts] float32: a wave a token
__global__ __launch_bounds__(MOE_ROUTE_TOKENS * TQK_WAVE)
void moe_choose_grouped_kernel(const float* __restrict__ logits, int n_tokens, int n_experts, int top, const float* __restrict__ correction, int n_groups, int keep,
                               float floor, int32_t* __restrict__ idx, float* __restrict__ weight) {
    __shared__ volatile float zs[MOE_ROUTE_TOKENS * MOE_MAX_EXPERTS], choices[MOE_ROUTE_TOKENS * MOE_MAX_EXPERTS], groups[MOE_ROUTE_TOKENS * MOE_MAX_EXPERTS];
    const int wave = threadIdx.x / TQK_WAVE, lane = threadIdx.x % TQK_WAVE;
    const int t = blockIdx.x * MOE_ROUTE_TOKENS + wave;
    if (t >= n_tokens) return;
    volatile float* z = zs + wave * MOE_MAX_EXPERTS;
    for (int e = lane; e < n_experts; e += TQK_WAVE) z[e] = logits[(size_t)t * n_experts + e];
    choose_grouped(z, choices + wave * MOE_MAX_EXPERTS, groups + wave * MOE_MAX_EXPERTS, n_experts, top, correction, n_groups, keep, floor, lane, idx + (size_t)t * top,
                   weight + (size_t)t * top);
}

// ---- group -----------------------------------------------------------------------------------
__global__ __launch_bounds__(1024)
void moe_group_kernel(const int32_t* __restrict__ idx, int n_pairs, int top, int n_experts, int tile_m, int32_t* __restrict__ pair_pos,
                      int32_t* __restrict__ sorted_tok, int32_t* __restrict__ tile_expert, int32_t* __restrict__ tile_row0,
                      int32_t* __restrict__ tile_rows, int32_t* __restrict__ n_tiles) {
    __shared__ int count[MOE_MAX_EXPERTS], offset[MOE_MAX_EXPERTS], tile_base[MOE_MAX_EXPERTS];
    for (int e = threadIdx.x; e < n_experts; e += blockDim.x) count[e] = 0;
    __syncthreads();
    for (int p = threadIdx.x; p < n_pairs; p += blockDim.x) {
        const int e = idx[p];
        pair_pos[p] = e < n_experts ? atomicAdd(&count[e], 1) : -1;
    }
    __syncthreads();
    if (threadIdx.x == 0) {
        int rows = 0, tiles = 0;
        for (int e = 0; e < n_experts; ++e) {
            offset[e] = rows;
            tile_base[e] = tiles;
            rows += count[e];
            tiles += (count[e] + tile_m - 1) / tile_m;
        }
        *n_tiles = tiles;
    }
    __syncthreads();
    for (int e = threadIdx.x; e < n_experts; e += blockDim.x) {
        const int n = count[e];
        for (int i = 0, tile = tile_base[e]; i < n; i += tile_m, ++tile) {
            tile_expert[tile] = e;
            tile_row0[tile] = offset[e] + i;
            tile_rows[tile] = min(tile_m, n - i);
        }
    }
    for (int p = threadIdx.x; p < n_pairs; p += blockDim.x) {
        const int e = idx[p];
        if (e >= n_experts) continue;
        const int row = offset[e] + pair_pos[p];
        pair_pos[p] = row;
        sorted_tok[row] = p / top;
    }
}

// ---- product ---------------------------------------------------------------------------------
// 32 rows x 64 features per block, 2 x 4 per thread, float32 fused multiply-adds in increasing k.
template <typename TX, typename TW, typename TY, bool GATED>
__global__ __launch_bounds__(256)
void moe_product_kernel(const TX* __restrict__ x, const int32_t* __restrict__ x_rows, const TW* __restrict__ w, long long expert_stride,
                        TY* __restrict__ y, int N, int K, int gate, float limit, float alpha, const int32_t* __restrict__ tile_expert,
                        const int32_t* __restrict__ tile_row0, const int32_t* __restrict__ tile_rows, const int32_t* __restrict__ n_tiles) {
    const int tile = blockIdx.y;
    if (tile >= *n_tiles) return;
    __shared__ float xs[MOE_TK][MOE_TM + 2];
    __shared__ float ws[GATED ? 2 : 1][MOE_TK][MOE_TN + 4];
    const int expert = tile_expert[tile], row0 = tile_row0[tile], n_rows = tile_rows[tile];
    const int n0 = blockIdx.x * MOE_TN;
    const TW* we = w + (size_t)expert * expert_stride;
    const int tid = threadIdx.x, tm = tid / 16, tn = tid % 16;
    float acc[GATED ? 2 : 1][2][4];
#pragma unroll
    for (int g = 0; g < (GATED ? 2 : 1); ++g)
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
            for (int j = 0; j < 4; ++j) acc[g][i][j] = 0.f;
    // the two x elements and the four weight elements a thread brings in per stage
    const int xr0 = tid / MOE_TK, xk = tid % MOE_TK;                // rows xr0 and xr0 + 16
    long long xsrc[2];
#pragma unroll
    for (int e = 0; e < 2; ++e) {
        const int r = xr0 + 16 * e;
        xsrc[e] = r < n_rows ? (long long)(x_rows ? x_rows[row0 + r] : row0 + r) * K : -1;
    }
    for (int k0 = 0; k0 < K; k0 += MOE_TK) {
#pragma unroll
        for (int e = 0; e < 2; ++e) xs[xk][xr0 + 16 * e] = (xsrc[e] >= 0 && k0 + xk < K) ? to_float(x[xsrc[e] + k0 + xk]) : 0.f;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int i = tid + e * 256, r = i / MOE_TK, kk = i % MOE_TK;
            const bool in = n0 + r < N && k0 + kk < K;
            ws[0][kk][r] = in ? to_float(we[(size_t)(n0 + r) * K + k0 + kk]) : 0.f;
            if (GATED) ws[GATED ? 1 : 0][kk][r] = in ? to_float(we[(size_t)(N + n0 + r) * K + k0 + kk]) : 0.f;
        }
        __syncthreads();
#pragma unroll
        for (int kk = 0; kk < MOE_TK; ++kk) {
            const float a0 = xs[kk][tm * 2], a1 = xs[kk][tm * 2 + 1];
#pragma unroll
            for (int g = 0; g < (GATED ? 2 : 1); ++g)
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    const float b = ws[g][kk][tn * 4 + j];
                    acc[g][0][j] = fmaf(a0, b, acc[g][0][j]);
                    acc[g][1][j] = fmaf(a1, b, acc[g][1][j]);
                }
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        const int r = tm * 2 + i;
        if (r >= n_rows) continue;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int n = n0 + tn * 4 + j;
            if (n >= N) continue;
            float v = acc[0][i][j];
            if (GATED) {
                // gate and up are rounded as stored products would be, then the gate in float32
                const float g = to_float(from_float<TY>(v)), u = to_float(from_float<TY>(acc[GATED ? 1 : 0][i][j]));
                v = gate_value(gate, limit, alpha, g, u);
            } else if (gate >= 0) {
                v = act_value(gate, limit, alpha, to_float(from_float<TY>(v)));
            }
            y[(size_t)(row0 + r) * N + n] = from_float<TY>(v);
        }
    }
}

// ---- combine ---------------------------------------------------------------------------------
struct CombineArgs {
    const void* y;
    const int32_t* pair_pos;
    const float* weight;
    int top;
    const void *x, *shared;         // x: the step's rows, for pairs without a row (or null); shared, beside: or null
    const float* shared_scale;
    const void* beside;
    float scale;
    void* out;                      // the sums, in the activation type; or, with h, the norm of the stream
    float* h;                       // null, or the stream, which the sums are added to
    const void* norm_w;
    float eps;
    int hidden;
};

template <typename TA> struct Four;
template <> struct Four<float> {
    __device__ static float4 load(const void* p, size_t at) { return *reinterpret_cast<const float4*>((const float*)p + at); }
    __device__ static void store(void* p, size_t at, float4 v) { *reinterpret_cast<float4*>((float*)p + at) = v; }
};
template <> struct Four<bf16_t> {
    __device__ static float4 load(const void* p, size_t at) {
        const uint2 u = *reinterpret_cast<const uint2*>((const bf16_t*)p + at);
        return make_float4(__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u), __uint_as_float(u.y << 16), __uint_as_float(u.y & 0xffff0000u));
    }
    __device__ static void store(void* p, size_t at, float4 v) {
        *reinterpret_cast<uint2*>((bf16_t*)p + at) = make_uint2(float_to_bf16_bits(v.x) | ((uint32_t)float_to_bf16_bits(v.y) << 16),
                                                               float_to_bf16_bits(v.z) | ((uint32_t)float_to_bf16_bits(v.w) << 16));
    }
};

// A block per token, four neighbouring elements a thread VPT times.  NORM: the sum goes to the stream h in float32, and out is the stream's RMS
// norm (h / rms(h) * norm_w), which the next layer reads.
template <typename TA, typename TW, int VPT, bool NORM>
__global__ __launch_bounds__(1024)
void moe_combine_vec_kernel(const CombineArgs a) {
    __shared__ int32_t row[MOE_MAX_EXPERTS];
    __shared__ float wt[MOE_MAX_EXPERTS];
    __shared__ float scratch[16];
    const size_t t = blockIdx.x;
    const int hidden = a.hidden, top = a.top;
    for (int k = threadIdx.x; k < top; k += blockDim.x) {
        row[k] = a.pair_pos[t * top + k];
        wt[k] = a.weight[t * top + k];
    }
    __syncthreads();
    const float ss = a.shared && a.shared_scale ? a.shared_scale[t] : 1.f;
    float4 keep[VPT];
    float sq = 0.f;
#pragma unroll
    for (int j = 0; j < VPT; ++j) {
        const int i = (j * blockDim.x + threadIdx.x) * 4;
        keep[j] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (i >= hidden) continue;
        float4 v = make_float4(0.f, 0.f, 0.f, 0.f), hv = v;
        if (NORM) hv = *reinterpret_cast<const float4*>(a.h + t * hidden + i);
#pragma unroll 4
        for (int k = 0; k < top; ++k) {
            const int r = row[k];
            const float4 u = Four<TA>::load(r >= 0 ? a.y : a.x, (r >= 0 ? (size_t)r : t) * hidden + i);
            const float w = wt[k];
            v.x = fmaf(w, u.x, v.x); v.y = fmaf(w, u.y, v.y); v.z = fmaf(w, u.z, v.z); v.w = fmaf(w, u.w, v.w);
        }
        if (a.shared) {
            const float4 u = Four<TA>::load(a.shared, t * hidden + i);
            v.x = fmaf(ss, u.x, v.x); v.y = fmaf(ss, u.y, v.y); v.z = fmaf(ss, u.z, v.z); v.w = fmaf(ss, u.w, v.w);
        }
        if (a.beside) {
            const float4 u = Four<TA>::load(a.beside, t * hidden + i);
            v.x += u.x; v.y += u.y; v.z += u.z; v.w += u.w;
        }
        if (!NORM) {
            Four<TA>::store(a.out, t * hidden + i, make_float4(v.x * a.scale, v.y * a.scale, v.z * a.scale, v.w * a.scale));
            continue;
        }
        hv.x = fmaf(a.scale, v.x, hv.x); hv.y = fmaf(a.scale, v.y, hv.y); hv.z = fmaf(a.scale, v.z, hv.z); hv.w = fmaf(a.scale, v.w, hv.w);
        *reinterpret_cast<float4*>(a.h + t * hidden + i) = hv;
        keep[j] = hv;
        sq += (hv.x * hv.x + hv.y * hv.y) + (hv.z * hv.z + hv.w * hv.w);
    }
    if (!NORM) return;
    const float rms = sqrtf(block_sum(sq, scratch) / (float)hidden + a.eps);
#pragma unroll
    for (int j = 0; j < VPT; ++j) {
        const int i = (j * blockDim.x + threadIdx.x) * 4;
        if (i >= hidden) continue;
        const float4 w = Four<TW>::load(a.norm_w, i), v = keep[j];
        Four<TA>::store(a.out, t * hidden + i, make_float4(v.x / rms * w.x, v.y / rms * w.y, v.z / rms * w.z, v.w / rms * w.w));
    }
}

// rows of any length and alignment, element by element
template <typename TA>
__global__ __launch_bounds__(256)
void moe_combine_kernel(const CombineArgs a) {
    // the token's rows and weights once, side by side, not one load after the other in front of every element
    __shared__ int32_t row[MOE_MAX_EXPERTS];
    __shared__ float wt[MOE_MAX_EXPERTS];
    const size_t t = blockIdx.x;
    const int hidden = a.hidden, top = a.top;
    for (int k = threadIdx.x; k < top; k += blockDim.x) {
        row[k] = a.pair_pos[t * top + k];
        wt[k] = a.weight[t * top + k];
    }
    __syncthreads();
    const float ss = a.shared && a.shared_scale ? a.shared_scale[t] : 1.f;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) {
        float v = 0.f;
#pragma unroll 4
        for (int k = 0; k < top; ++k) {
            const int r = row[k];
            v = fmaf(wt[k], to_float(((const TA*)(r >= 0 ? a.y : a.x))[(r >= 0 ? (size_t)r : t) * hidden + i]), v);
        }
        if (a.shared) v = fmaf(ss, to_float(((const TA*)a.shared)[t * hidden + i]), v);
        if (a.beside) v += to_float(((const TA*)a.beside)[t * hidden + i]);
        ((TA*)a.out)[t * hidden + i] = from_float<TA>(v * a.scale);
    }
}

// ---- scale -----------------------------------------------------------------------------------
template <typename TA>
__global__ __launch_bounds__(256)
void moe_scale_rows_kernel(const TA* __restrict__ x, const int32_t* __restrict__ pair_pos, const float* __restrict__ weight, int top,
                           TA* __restrict__ rows, float* __restrict__ unit, int hidden) {
    const size_t p = blockIdx.x;
    const float w = weight[p];
    const TA* src = x + (p / top) * hidden;
    const int row = pair_pos[p];
    if (threadIdx.x == 0) unit[p] = row < 0 ? w : 1.f;              // without a row: the input itself, times the weight
    if (row < 0) return;
    TA* dst = rows + (size_t)row * hidden;
    for (int i = threadIdx.x; i < hidden; i += blockDim.x) dst[i] = from_float<TA>(w * to_float(src[i]));
}

// ---- entry points ----------------------------------------------------------------------------
extern "C" int tqk_moe_scale_rows(const void* x, int act_dtype, const int32_t* pair_pos, const float* weight, int top, void* rows, float* unit,
                                  int n_tokens, int hidden, void* stream) {
    TQK_REQUIRE(x && pair_pos && weight && rows && unit, "tqk_moe_scale_rows: null pointer");
    TQK_REQUIRE(top > 0 && hidden > 0 && n_tokens >= 0 && (long long)n_tokens * top <= 0x7fffffff, "tqk_moe_scale_rows: bad sizes");
    if (n_tokens == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    const unsigned pairs = (unsigned)(n_tokens * top);
    if (act_dtype == TQK_F32) moe_scale_rows_kernel<float><<<pairs, 256, 0, s>>>((const float*)x, pair_pos, weight, top, (float*)rows, unit, hidden);
    else if (act_dtype == TQK_BF16) moe_scale_rows_kernel<bf16_t><<<pairs, 256, 0, s>>>((const bf16_t*)x, pair_pos, weight, top, (bf16_t*)rows, unit, hidden);
    else return tqk_fail("tqk_moe_scale_rows: unknown dtype %d", act_dtype);
    return tqk_check_launch("tqk_moe_scale_rows");
}

extern "C" int tqk_moe_max_experts(void) { return MOE_MAX_EXPERTS; }
extern "C" int tqk_moe_tile_rows(void) { return MOE_TM; }
extern "C" int tqk_moe_max_tiles(int n_pairs, int n_experts, int tile_m) { return (n_pairs + tile_m - 1) / tile_m + n_experts; }

extern "C" int tqk_moe_route(const void* x, int act_dtype, const void* w_router, int w_dtype, int n_experts, int hidden, int top, float scale,
                             int mode, int32_t* idx, float* weight, const void* gate_w, float* gate_out, int n_tokens, void* stream) {
    TQK_REQUIRE(x && w_router && idx && weight, "tqk_moe_route: null pointer");
    TQK_REQUIRE(n_experts > 0 && n_experts <= MOE_MAX_EXPERTS, "tqk_moe_route: %d experts, the kernel takes 1 to %d", n_experts, MOE_MAX_EXPERTS);
    TQK_REQUIRE(top > 0 && top <= n_experts && hidden > 0 && n_tokens >= 0, "tqk_moe_route: bad sizes (top %d of %d experts)", top, n_experts);
    TQK_REQUIRE(!gate_w || gate_out, "tqk_moe_route: a gate without a place for its values");
    if (n_tokens == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
#define TQK_ROUTE(TA, TW) \
    do { if (n_tokens >= 512) moe_route_kernel<TA, TW, MOE_ROUTE_TOKENS><<<(n_tokens + MOE_ROUTE_TOKENS - 1) / MOE_ROUTE_TOKENS, MOE_ROUTE_WAVES * TQK_WAVE, 0, s>>>((const TA*)x, n_tokens, (const TW*)w_router, n_experts, hidden, top, scale, mode, idx, weight, (const TW*)gate_w, gate_out); \
        else moe_route_kernel<TA, TW, 1><<<n_tokens, MOE_ROUTE_WAVES * TQK_WAVE, 0, s>>>((const TA*)x, n_tokens, (const TW*)w_router, n_experts, hidden, top, scale, mode, idx, weight, (const TW*)gate_w, gate_out); } while (0)
    if (act_dtype == TQK_F32 && w_dtype == TQK_F32) TQK_ROUTE(float, float);
    else if (act_dtype == TQK_F32 && w_dtype == TQK_BF16) TQK_ROUTE(float, bf16_t);
    else if (act_dtype == TQK_BF16 && w_dtype == TQK_F32) TQK_ROUTE(bf16_t, float);
    else if (act_dtype == TQK_BF16 && w_dtype == TQK_BF16) TQK_ROUTE(bf16_t, bf16_t);
    else return tqk_fail("tqk_moe_route: unknown dtypes %d, %d", act_dtype, w_dtype);
#undef TQK_ROUTE
    return tqk_check_launch("tqk_moe_route");
}

extern "C" int tqk_moe_route_grouped(const void* x, int act_dtype, const void* w_router, int w_dtype, int n_experts, int hidden, int top, const float* correction,
                                     int n_groups, int keep, float floor, int32_t* idx, float* weight, int n_tokens, void* stream) {
    TQK_REQUIRE(x && w_router && idx && weight, "tqk_moe_route_grouped: null pointer");
    TQK_REQUIRE(n_experts > 0 && n_experts <= MOE_MAX_EXPERTS, "tqk_moe_route_grouped: %d experts, the kernel takes 1 to %d", n_experts, MOE_MAX_EXPERTS);
    TQK_REQUIRE(n_groups > 0 && n_experts % n_groups == 0 && keep > 0 && keep <= n_groups, "tqk_moe_route_grouped: %d of %d groups of %d experts", keep, n_groups, n_experts);
    TQK_REQUIRE(top > 0 && top <= keep * (n_experts / n_groups) && hidden > 0 && n_tokens >= 0, "tqk_moe_route_grouped: bad sizes (top %d of %d experts)", top,
                keep * (n_experts / n_groups));
    if (n_tokens == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
#define TQK_ROUTE(TA, TW) \
    do { if (n_tokens >= 512) moe_route_grouped_kernel<TA, TW, MOE_ROUTE_TOKENS><<<(n_tokens + MOE_ROUTE_TOKENS - 1) / MOE_ROUTE_TOKENS, MOE_ROUTE_WAVES * TQK_WAVE, 0, s>>>((const TA*)x, n_tokens, (const TW*)w_router, n_experts, hidden, top, correction, n_groups, keep, floor, idx, weight); \
        else moe_route_grouped_kernel<TA, TW, 1><<<n_tokens, MOE_ROUTE_WAVES * TQK_WAVE, 0, s>>>((const TA*)x, n_tokens, (const TW*)w_router, n_experts, hidden, top, correction, n_groups, keep, floor, idx, weight); } while (0)
    if (act_dtype == TQK_F32 && w_dtype == TQK_F32) TQK_ROUTE(float, float);
    else if (act_dtype == TQK_F32 && w_dtype == TQK_BF16) TQK_ROUTE(float, bf16_t);
    else if (act_dtype == TQK_BF16 && w_dtype == TQK_F32) TQK_ROUTE(bf16_t, float);
    else if (act_dtype == TQK_BF16 && w_dtype == TQK_BF16) TQK_ROUTE(bf16_t, bf16_t);
    else return tqk_fail("tqk_moe_route_grouped: unknown dtypes %d, %d", act_dtype, w_dtype);
#undef TQK_ROUTE
    return tqk_check_launch("tqk_moe_route_grouped");
}

extern "C" int tqk_moe_choose_grouped(const float* logits, int n_experts, int top, const float* correction, int n_groups, int keep, float floor, int32_t* idx,
                                      float* weight, int n_tokens, void* stream) {
    TQK_REQUIRE(logits && idx && weight, "tqk_moe_choose_grouped: null pointer");
    TQK_REQUIRE(n_experts > 0 && n_experts <= MOE_MAX_EXPERTS, "tqk_moe_choose_grouped: %d experts, the kernel takes 1 to %d", n_experts, MOE_MAX_EXPERTS);
    TQK_REQUIRE(n_groups > 0 && n_experts % n_groups == 0 && keep > 0 && keep <= n_groups && top > 0 && top <= keep * (n_experts / n_groups) && n_tokens >= 0,
                "tqk_moe_choose_grouped: top %d of %d of %d groups of %d experts", top, keep, n_groups, n_experts);
    if (n_tokens == 0) return 0;
    moe_choose_grouped_kernel<<<(n_tokens + MOE_ROUTE_TOKENS - 1) / MOE_ROUTE_TOKENS, MOE_ROUTE_TOKENS * TQK_WAVE, 0, (hipStream_t)stream>>>(
        logits, n_tokens, n_experts, top, correction, n_groups, keep, floor, idx, weight);
    return tqk_check_launch("tqk_moe_choose_grouped");
}

extern "C" int tqk_moe_group(const int32_t* idx, int n_tokens, int top, int n_experts, int tile_m, int32_t* pair_pos, int32_t* sorted_tok,
                             int32_t* tile_expert, int32_t* tile_row0, int32_t* tile_rows, int32_t* n_tiles, void* stream) {
    TQK_REQUIRE(idx && pair_pos && sorted_tok && tile_expert && tile_row0 && tile_rows && n_tiles, "tqk_moe_group: null pointer");
    TQK_REQUIRE(n_experts > 0 && n_experts <= MOE_MAX_EXPERTS && top > 0 && n_tokens >= 0, "tqk_moe_group: bad sizes");
    TQK_REQUIRE((long long)n_tokens * top <= 0x7fffffff, "tqk_moe_group: too many pairs");
    TQK_REQUIRE(tile_m > 0, "tqk_moe_group: tiles of %d rows", tile_m);
    if (n_tokens == 0) return 0;
    moe_group_kernel<<<1, 1024, 0, (hipStream_t)stream>>>(idx, n_tokens * top, top, n_experts, tile_m, pair_pos, sorted_tok, tile_expert, tile_row0,
                                                          tile_rows, n_tiles);
    return tqk_check_launch("tqk_moe_group");
}

template <typename TX, typename TW, typename TY>
static int launch_moe_product(const void* x, const int32_t* x_rows, const void* w, long long expert_stride, void* y, int N, int K, int gated,
                              int gate, float limit, float alpha, const int32_t* tile_expert, const int32_t* tile_row0,
                              const int32_t* tile_rows, const int32_t* n_tiles, int max_tiles, hipStream_t s) {
    dim3 grid((N + MOE_TN - 1) / MOE_TN, max_tiles);
    if (gated == 1)
        moe_product_kernel<TX, TW, TY, true><<<grid, 256, 0, s>>>((const TX*)x, x_rows, (const TW*)w, expert_stride, (TY*)y, N, K, gate, limit, alpha,
                                                                  tile_expert, tile_row0, tile_rows, n_tiles);
    else
        moe_product_kernel<TX, TW, TY, false><<<grid, 256, 0, s>>>((const TX*)x, x_rows, (const TW*)w, expert_stride, (TY*)y, N, K, gated == 2 ? gate : -1, limit, alpha,
                                                                   tile_expert, tile_row0, tile_rows, n_tiles);
    return tqk_check_launch("tqk_moe_product");
}

extern "C" int tqk_moe_product(const void* x, int act_dtype, const int32_t* x_rows, const void* w, int w_dtype, long long expert_stride, void* y,
                               int N, int K, int gated, int gate, float limit, float alpha, const int32_t* tile_expert,
                               const int32_t* tile_row0, const int32_t* tile_rows, const int32_t* n_tiles, int max_tiles, void* stream) {
    TQK_REQUIRE(x && w && y && tile_expert && tile_row0 && tile_rows && n_tiles, "tqk_moe_product: null pointer");
    TQK_REQUIRE(N > 0 && K > 0 && max_tiles >= 0 && max_tiles <= 65535, "tqk_moe_product: bad sizes (N %d, K %d, %d tiles)", N, K, max_tiles);
    TQK_REQUIRE(gated >= 0 && gated <= 2, "tqk_moe_product: gated must be 0 (plain), 1 (gate and up) or 2 (one product with its activation), got %d", gated);
    TQK_REQUIRE(!gated || (gate >= 0 && gate < TQK_GATE_KINDS), "tqk_moe_product: unknown gate %d", gate);
    TQK_REQUIRE(expert_stride >= (long long)(gated == 1 ? 2 : 1) * N * K, "tqk_moe_product: experts overlap");
    /* the tile lists must have been made for tiles of tqk_moe_tile_rows() rows */
    if (max_tiles == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
#define TQK_MOE(TX, TW) \
    return launch_moe_product<TX, TW, TX>(x, x_rows, w, expert_stride, y, N, K, gated, gate, limit, alpha, tile_expert, tile_row0, tile_rows, n_tiles, max_tiles, s)
    if (act_dtype == TQK_F32 && w_dtype == TQK_F32) TQK_MOE(float, float);
    if (act_dtype == TQK_F32 && w_dtype == TQK_BF16) TQK_MOE(float, bf16_t);
    if (act_dtype == TQK_BF16 && w_dtype == TQK_F32) TQK_MOE(bf16_t, float);
    if (act_dtype == TQK_BF16 && w_dtype == TQK_BF16) TQK_MOE(bf16_t, bf16_t);
#undef TQK_MOE
    return tqk_fail("tqk_moe_product: unknown dtypes %d, %d", act_dtype, w_dtype);
}

static int combine_args(CombineArgs& a, const void* y, const int32_t* pair_pos, const float* weight, int top, const void* x, const void* shared,
                        const float* shared_scale, const void* beside, float scale, void* out, int n_tokens, int hidden) {
    TQK_REQUIRE(y && pair_pos && weight && out, "tqk_moe_combine: null pointer");
    TQK_REQUIRE(top > 0 && top <= MOE_MAX_EXPERTS && hidden > 0 && n_tokens >= 0, "tqk_moe_combine: bad sizes");
    // (without x no pair may be without a row: every pair_pos is then a row of y)
    a = {y, pair_pos, weight, top, x ? x : y, shared, shared_scale, beside, scale, out, nullptr, nullptr, 0.f, hidden};
    return 0;
}
// rows in pieces of four elements, each piece at its alignment; a thread takes up to two of them
static bool combine_in_pieces(const CombineArgs& a) {
    return a.hidden % 4 == 0 && a.hidden <= 8192 &&
           ((((uintptr_t)a.y | (uintptr_t)a.x | (uintptr_t)a.shared | (uintptr_t)a.beside | (uintptr_t)a.out | (uintptr_t)a.h | (uintptr_t)a.norm_w)) & 15) == 0;
}
template <typename TA, typename TW, bool NORM>
static void launch_combine(const CombineArgs& a, int n_tokens, hipStream_t s) {
    const int pieces = a.hidden / 4;
    const int threads = pieces >= 1024 ? 1024 : (pieces + TQK_WAVE - 1) / TQK_WAVE * TQK_WAVE;
    if (pieces <= threads) moe_combine_vec_kernel<TA, TW, 1, NORM><<<n_tokens, threads, 0, s>>>(a);
    else moe_combine_vec_kernel<TA, TW, 2, NORM><<<n_tokens, threads, 0, s>>>(a);
}

extern "C" int tqk_moe_combine(const void* y, int act_dtype, const int32_t* pair_pos, const float* weight, int top, const void* x, const void* shared,
                               const float* shared_scale, const void* beside, float scale, void* out, int n_tokens, int hidden, void* stream) {
    CombineArgs a;
    if (combine_args(a, y, pair_pos, weight, top, x, shared, shared_scale, beside, scale, out, n_tokens, hidden)) return -1;
    TQK_REQUIRE(act_dtype == TQK_F32 || act_dtype == TQK_BF16, "tqk_moe_combine: unknown dtype %d", act_dtype);
    if (n_tokens == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    if (combine_in_pieces(a)) {
        if (act_dtype == TQK_F32) launch_combine<float, float, false>(a, n_tokens, s);
        else launch_combine<bf16_t, float, false>(a, n_tokens, s);
    } else if (act_dtype == TQK_F32) moe_combine_kernel<float><<<n_tokens, 256, 0, s>>>(a);
    else moe_combine_kernel<bf16_t><<<n_tokens, 256, 0, s>>>(a);
    return tqk_check_launch("tqk_moe_combine");
}

extern "C" int tqk_moe_combine_norm_supported(int hidden) { return hidden > 0 && hidden % 4 == 0 && hidden <= 8192; }

extern "C" int tqk_moe_combine_norm(float* h, const void* y, int act_dtype, const int32_t* pair_pos, const float* weight, int top, const void* x,
                                    const void* shared, const float* shared_scale, const void* beside, float scale, const void* norm_w, int norm_w_dtype,
                                    float eps, void* out, int n_tokens, int hidden, void* stream) {
    CombineArgs a;
    if (combine_args(a, y, pair_pos, weight, top, x, shared, shared_scale, beside, scale, out, n_tokens, hidden)) return -1;
    TQK_REQUIRE(h && norm_w, "tqk_moe_combine_norm: null pointer");
    a.h = h; a.norm_w = norm_w; a.eps = eps;
    TQK_REQUIRE(combine_in_pieces(a), "tqk_moe_combine_norm: rows of %d elements, or operands that are not aligned", hidden);
    if (n_tokens == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    if (act_dtype == TQK_F32 && norm_w_dtype == TQK_F32) launch_combine<float, float, true>(a, n_tokens, s);
    else if (act_dtype == TQK_F32 && norm_w_dtype == TQK_BF16) launch_combine<float, bf16_t, true>(a, n_tokens, s);
    else if (act_dtype == TQK_BF16 && norm_w_dtype == TQK_F32) launch_combine<bf16_t, float, true>(a, n_tokens, s);
    else if (act_dtype == TQK_BF16 && norm_w_dtype == TQK_BF16) launch_combine<bf16_t, bf16_t, true>(a, n_tokens, s);
    else return tqk_fail("tqk_moe_combine_norm: unknown dtypes %d, %d", act_dtype, norm_w_dtype);
    return tqk_check_launch("tqk_moe_combine_norm");
}
