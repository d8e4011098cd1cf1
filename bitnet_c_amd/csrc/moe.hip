// A mixture-of-experts feed-forward.  Expert e is  W_down[e] act(W_up[e] x)  (no gate), or, in the gated form,
// W_down[e] glu(W_gate[e] x, W_up[e] x)  with the clamped unit  glu(g, u) = g' sigmoid(slope g') (u' + shift),
// g' = min(g, limit), u' = clamp(u, -limit, limit)  (gate and up rows stacked, [E, 2 F, D]).
//
//   bn_moe_route     router logits z = W_r h (+ a bias per expert) in float32 (one workgroup a token), scores sigmoid(z) or softmax(z), the top_k
//                    largest (ties: the lower index; with a choice bias the largest score + bias, the weights staying the
//                    plain scores), optionally divided by their sum (+ floor), times a constant -> expert ids and weights
//                    [T, top_k]; optionally also sigmoid(w_g . h) per token, the gate of a shared expert.  With groups the
//                    experts fall into groups of neighbours, a group ranks by its best member, and only members of the
//                    best `keep` groups (ties: the lower index) can be chosen
//   bn_gated_unit    rows of stacked (gate | up) products -> the clamped unit, optionally times a factor per row
//   bn_moe_experts   for every (token, choice) pair: y = W_down[e] act(W_up[e] (w h)) when the weight multiplies the
//                    expert's input, w * W_down[e] act(W_up[e] h) when it multiplies the output; a pair reads its expert's
//                    two matrices once, their rows spread over workgroups.  The products accumulate in float32; the scaled
//                    input and the hidden vector are rounded to the activations' type as a product of that type would
//                    see them.
//   bn_moe_group     (bf16, steps of many rows) pairs ordered by expert, tiles of rows of one expert each, and the inputs
//                    gathered in that order, for the grouped matrix products of gemm_mfma.hip
// Experts from E on are identity experts: they have no matrices, and their output is the token's own row times the weight.
// The outputs of a token's choices land in slab j of y [top_k, T, D] (float32) and are added by whoever consumes y.
#include "common.h"
#include <math.h>

#define MOE_MAX_EXPERTS 1024
#define MOE_SCORE_SIGMOID 0
#define MOE_SCORE_SOFTMAX 1

struct RouteArgs {
    const void* h;            // [T, ld]
    const float* wr;          // [E, D] float32
    int* ids;                 // [T, K]
    float* wts;               // [T, K]
    int ld, T, D, E, K, scoring, renorm;
    const float* bias;        // [E] added to the scores for the choice alone; null: the choice goes by the scores
    const float* zbias;       // [E] added to the logits themselves (a router with a bias); null: none
    const float* gate_w;      // [D]: gate_out[t] = sigmoid(gate_w . h); null: none
    float* gate_out;          // [T]
    float floor, scale;       // weights = score / (sum of the chosen + floor) (when renorm) * scale
    int groups, keep;         // groups > 1: E / groups neighbours a group, the best `keep` groups stay in the choice
};

// A wave an expert as far as a workgroup's 16 waves go.  Steps of few rows (MOE_ROUTE_FEW_ROWS): a workgroup a token.  Steps
// of many: four tokens a workgroup, whose rows lie in shared memory and whose waves read a router row once for all four and
// then choose for a token each.  A token's sums have one order either way.
#define MOE_ROUTE_FEW_ROWS 256
#define MOE_ROUTE_THREADS 1024
#define MOE_ROUTE_TOKENS 4

__device__ __forceinline__ float4 moe_load4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 moe_load4(const bf16* p) {
    const uint2 t = *reinterpret_cast<const uint2*>(p);
    return make_float4(bf16lo_to_f32(t.x), bf16hi_to_f32(t.x), bf16lo_to_f32(t.y), bf16hi_to_f32(t.y));
}

__host__ __device__ __forceinline__ int moe_route_row_bytes(int D, int elt) { return (D * elt + 15) & ~15; }

// The waves take the experts in turn (a row of the router as 16-byte loads across the lanes with the tokens' rows beside it,
// several in flight); then wave i chooses for token i.  PL: experts a lane of such a wave holds, E <= 64 PL; TK: tokens of the
// workgroup, which has at least as many waves.
template <typename T, int PL, int TK>
__global__ __launch_bounds__(MOE_ROUTE_THREADS, PL == 1 ? 8 : 4) void moe_route_kernel(RouteArgs a) {
    // the tokens' rows (TK > 1; whole 16-byte groups a row), then per token the experts' logits and the groups' best values
    extern __shared__ __align__(16) unsigned char route_raw[];
    const int t0 = blockIdx.x * TK, lane = threadIdx.x & (BN_WAVE - 1), wave = threadIdx.x / BN_WAVE;
    const T* h[TK];
#pragma unroll
    for (int k = 0; k < TK; ++k) h[k] = reinterpret_cast<const T*>(a.h) + (size_t)min(t0 + k, a.T - 1) * a.ld;
    const bool whole = a.D % 4 == 0 && (TK > 1 || (a.ld % 4 == 0 && ((uintptr_t)a.h & (4 * sizeof(T) - 1)) == 0));
    const int row_bytes = TK > 1 ? moe_route_row_bytes(a.D, (int)sizeof(T)) : 0;
    float* route_smem = reinterpret_cast<float*>(route_raw + TK * row_bytes);
    if (TK > 1) {
#pragma unroll
        for (int k = 0; k < TK; ++k) {
            T* hs = reinterpret_cast<T*>(route_raw + k * row_bytes);
            if (a.ld * sizeof(T) % 16 == 0 && a.D * sizeof(T) % 16 == 0 && ((uintptr_t)a.h & 15) == 0) {
                for (int d = threadIdx.x; d < (int)(a.D * sizeof(T) / 16); d += blockDim.x)
                    reinterpret_cast<uint4*>(hs)[d] = reinterpret_cast<const uint4*>(h[k])[d];
            } else {
                for (int d = threadIdx.x; d < a.D; d += blockDim.x) hs[d] = h[k][d];
            }
            h[k] = hs;
        }
        __syncthreads();
    }
    // the shared expert's gate is one more row: it takes its turn among the waves after the experts
    for (int e = wave; e < a.E + (a.gate_w ? 1 : 0); e += blockDim.x / BN_WAVE) {
        const float* w = e < a.E ? a.wr + (size_t)e * a.D : a.gate_w;
        float s[TK];
#pragma unroll
        for (int k = 0; k < TK; ++k) s[k] = 0.f;
        if (whole) {
#pragma unroll(TK == 1 ? 8 : 2)
            for (int d = 4 * lane; d < a.D; d += 4 * BN_WAVE) {
                const float4 wv = *reinterpret_cast<const float4*>(w + d);
#pragma unroll
                for (int k = 0; k < TK; ++k) {
                    const float4 xv = moe_load4(h[k] + d);
                    s[k] = fmaf(xv.x, wv.x, s[k]); s[k] = fmaf(xv.y, wv.y, s[k]);
                    s[k] = fmaf(xv.z, wv.z, s[k]); s[k] = fmaf(xv.w, wv.w, s[k]);
                }
            }
        } else {
            for (int d = lane; d < a.D; d += BN_WAVE)
#pragma unroll
                for (int k = 0; k < TK; ++k) s[k] = fmaf(to_f32(h[k][d]), w[d], s[k]);
        }
#pragma unroll
        for (int k = 0; k < TK; ++k) {
            s[k] = wave_sum(s[k]);
            if (lane == 0) {
                if (e < a.E) route_smem[k * (a.E + a.groups) + e] = a.zbias ? s[k] + a.zbias[e] : s[k];
                else if (t0 + k < a.T) a.gate_out[t0 + k] = 1.0f / (1.0f + expf(-s[k]));
            }
        }
    }
    __syncthreads();
    const int t = t0 + wave;
    if (wave >= TK || t >= a.T) return;
    float* zs = route_smem + wave * (a.E + a.groups);
    float z[PL];                               // expert lane + 64 j
#pragma unroll
    for (int j = 0; j < PL; ++j) z[j] = lane + BN_WAVE * j < a.E ? zs[lane + BN_WAVE * j] : -INFINITY;
    float zmax = -INFINITY, denom = 1.f;
    if (a.scoring == MOE_SCORE_SOFTMAX) {
#pragma unroll
        for (int j = 0; j < PL; ++j) zmax = fmaxf(zmax, z[j]);
        zmax = wave_max(zmax);
        float sum = 0.f;
#pragma unroll
        for (int j = 0; j < PL; ++j) sum += z[j] == -INFINITY ? 0.f : expf(z[j] - zmax);
        denom = wave_sum(sum);
    }
    // with a choice bias the experts are ranked by score + bias: the scores of all experts are formed first and z holds
    // the ranking value from here on
    float sc[PL];
    if (a.bias) {
#pragma unroll
        for (int j = 0; j < PL; ++j) {
            const int e = lane + BN_WAVE * j;
            sc[j] = 0.f;
            if (e < a.E) {
                sc[j] = a.scoring == MOE_SCORE_SOFTMAX ? expf(z[j] - zmax) / denom : 1.0f / (1.0f + expf(-z[j]));
                z[j] = sc[j] + a.bias[e];
            }
        }
    }
    if (a.groups > 1) {
        // the ranking values (the logits rank as their scores do) meet in the wave's own part of shared memory: a lane
        // takes groups lane, lane + 64, ..., forms their best members' values, then counts the groups ahead of each
        float* rank = zs;
        float* best = zs + a.E;
        const int size = a.E / a.groups;
#pragma unroll
        for (int j = 0; j < PL; ++j)
            if (lane + BN_WAVE * j < a.E) rank[lane + BN_WAVE * j] = z[j];
        __threadfence_block();
        __builtin_amdgcn_wave_barrier();
        for (int g = lane; g < a.groups; g += BN_WAVE) {
            float m = -INFINITY;
            for (int i = 0; i < size; ++i) m = fmaxf(m, rank[g * size + i]);
            best[g] = m;
        }
        __threadfence_block();
        __builtin_amdgcn_wave_barrier();
#pragma unroll
        for (int j = 0; j < PL; ++j) {
            const int e = lane + BN_WAVE * j;
            if (e >= a.E) continue;
            const int g = e / size;
            const float m = best[g];
            int ahead = 0;
            for (int o = 0; o < a.groups; ++o) ahead += (best[o] > m || (best[o] == m && o < g)) ? 1 : 0;
            if (ahead >= a.keep) z[j] = -INFINITY;
        }
    }
    float total = 0.f, mine_w = 0.f;
    int mine_id = 0;
    for (int k = 0; k < a.K; ++k) {
        float best = -INFINITY;
        int at = MOE_MAX_EXPERTS;
#pragma unroll
        for (int j = 0; j < PL; ++j)
            if (z[j] > best) { best = z[j]; at = lane + BN_WAVE * j; }
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) {
            const float ob = __shfl_xor(best, o, BN_WAVE);
            const int oa = __shfl_xor(at, o, BN_WAVE);
            if (ob > best || (ob == best && oa < at)) { best = ob; at = oa; }
        }
        if (at >= a.E) at = k;                           // a row of NaNs (a padding row's garbage): still an expert that exists
        float own = 0.f;                                 // the chosen expert's plain score, held by the lane that owns it
#pragma unroll
        for (int j = 0; j < PL; ++j)
            if (at == lane + BN_WAVE * j) { z[j] = -INFINITY; if (a.bias) own = sc[j]; }
        const float score = a.bias ? wave_sum(own)
                          : a.scoring == MOE_SCORE_SOFTMAX ? expf(best - zmax) / denom : 1.0f / (1.0f + expf(-best));
        total += score;
        if (lane == k % BN_WAVE && k < BN_WAVE) { mine_w = score; mine_id = at; }
        if (k >= BN_WAVE && lane == 0) {                  // more choices than lanes: stored as they come
            a.ids[(size_t)t * a.K + k] = at;
            a.wts[(size_t)t * a.K + k] = score;
        }
    }
    const float norm = (a.renorm ? 1.0f / (total + a.floor) : 1.0f) * a.scale;
    if (lane < a.K) {
        a.ids[(size_t)t * a.K + lane] = mine_id;
        a.wts[(size_t)t * a.K + lane] = mine_w * norm;
    }
    if ((a.renorm || a.scale != 1.0f) && a.K > BN_WAVE && lane == 0)
        for (int k = BN_WAVE; k < a.K; ++k) a.wts[(size_t)t * a.K + k] *= norm;
}

extern "C" int bn_moe_route(int dtype, const void* h, int ld, const float* wr, int* ids, float* wts, int n_tokens, int D, int E,
                            int K, int scoring, int renorm, const float* bias, float floor, float scale, const float* gate_w,
                            float* gate_out, const float* zbias, int groups, int keep, hipStream_t s) {
    // groups of equal size, of which the kept ones hold at least the chosen number
    if (groups < 1 || E % groups || keep < 1 || keep > groups || (long long)keep * (E / groups) < K) return BN_ERR_ARG;
    if ((gate_w == nullptr) != (gate_out == nullptr) || ((uintptr_t)gate_w & 15) || !(floor >= 0.f)) return BN_ERR_ARG;
    if (n_tokens <= 0 || D <= 0 || E <= 0 || E > MOE_MAX_EXPERTS || K <= 0 || K > E || ld < D || !h || !wr || !ids || !wts)
        return BN_ERR_ARG;
    if (scoring != MOE_SCORE_SIGMOID && scoring != MOE_SCORE_SOFTMAX) return BN_ERR_ARG;
    if ((uintptr_t)wr & 15) return BN_ERR_ARG;
    RouteArgs a;
    a.h = h; a.wr = wr; a.ids = ids; a.wts = wts; a.ld = ld; a.T = n_tokens; a.D = D; a.E = E; a.K = K; a.scoring = scoring; a.renorm = renorm ? 1 : 0;
    a.bias = bias; a.zbias = zbias; a.gate_w = gate_w; a.gate_out = gate_out; a.floor = floor; a.scale = scale;
    a.groups = groups; a.keep = keep;
    if (dtype != BN_DT_F32 && dtype != BN_DT_BF16) return BN_ERR_DTYPE;
    const size_t rows = (size_t)MOE_ROUTE_TOKENS * moe_route_row_bytes(D, dtype == BN_DT_F32 ? 4 : 2);
    const bool few = n_tokens <= MOE_ROUTE_FEW_ROWS || rows + (size_t)MOE_ROUTE_TOKENS * (E + groups) * sizeof(float) > 64 * 1024;
    const int tk = few ? 1 : MOE_ROUTE_TOKENS;
    const size_t shm = (few ? 0 : rows) + (size_t)tk * (E + groups) * sizeof(float);
    const dim3 grid((n_tokens + tk - 1) / tk), block(E > 4 ? MOE_ROUTE_THREADS : 4 * BN_WAVE);
#define MOE_ROUTE_GO(PL_)                                                                                                   \
    do {                                                                                                                    \
        if (few && dtype == BN_DT_F32) hipLaunchKernelGGL((moe_route_kernel<float, PL_, 1>), grid, block, shm, s, a);       \
        else if (few) hipLaunchKernelGGL((moe_route_kernel<bf16, PL_, 1>), grid, block, shm, s, a);                         \
        else if (dtype == BN_DT_F32) hipLaunchKernelGGL((moe_route_kernel<float, PL_, MOE_ROUTE_TOKENS>), grid, block, shm, s, a); \
        else hipLaunchKernelGGL((moe_route_kernel<bf16, PL_, MOE_ROUTE_TOKENS>), grid, block, shm, s, a);                   \
    } while (0)
    if (E <= BN_WAVE) MOE_ROUTE_GO(1);
    else if (E <= 4 * BN_WAVE) MOE_ROUTE_GO(4);
    else MOE_ROUTE_GO(MOE_MAX_EXPERTS / BN_WAVE);
#undef MOE_ROUTE_GO
    return bn_launch_status();
}

// ---- a (token, choice) pair at a time ----------------------------------------------------------------------------------
// Steps of few rows: every pair reads its expert's two matrices once, and the rows of a matrix are spread over many
// workgroups so that one pair alone fills the chip (two launches: the hidden vector, then the output).  A workgroup stages
// the pair's input vector in shared memory as float32, each of its waves takes MOE_PAIR_ROWS / 4 rows of the matrix, a row
// as 16-byte loads across the lanes (bf16 rows of whole 8-element groups) or element by element, and sums in float32.
#define MOE_PAIR_THREADS 256
#define MOE_PAIR_ROWS 8

struct PairArgs {
    const void* h;            // [T, ld]
    const void* w_up;         // [E, F, D]
    const void* w_down;       // [E, D, F]
    const int* ids;           // [T, K]
    const float* wts;         // [T, K]
    float* hidden;            // [T K, F] float32 holding values of the activations' type
    float* y;                 // [K, T, D]
    int ld, T, D, F, K, E, act, weight_on_input;   // T: the rows of a slab of y; ids from E on: identity experts
    int gated;                // w_up is [E, 2 F, D]: F gate rows, then F up rows; hidden = the clamped unit of the two
    float limit, slope, shift;
};

// the clamped gated unit: g' sigmoid(slope g') (u' + shift), g' = min(g, limit), u' = clamp(u, -limit, limit)
__device__ __forceinline__ float moe_clamped_unit(float g, float u, float limit, float slope, float shift) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g / (1.0f + expf(-slope * g)) * (u + shift);
}

// sum over n of x[i] w[i]: x in shared memory, w a row in global memory; every lane gets the sum
template <typename T>
__device__ __forceinline__ float moe_row_dot(const T* __restrict__ w, const float* __restrict__ x, int n, int lane) {
    float s = 0.f;
    for (int i = lane; i < n; i += BN_WAVE) s = fmaf(x[i], to_f32(w[i]), s);
    return wave_sum(s);
}
template <>
__device__ __forceinline__ float moe_row_dot<bf16>(const bf16* __restrict__ w, const float* __restrict__ x, int n, int lane) {
    float s = 0.f;
    if (n % 8 == 0 && ((uintptr_t)w & 15) == 0) {
#pragma unroll 4
        for (int i = 8 * lane; i < n; i += 8 * BN_WAVE) {
            const uint4 p = *reinterpret_cast<const uint4*>(w + i);
            const float4 a = *reinterpret_cast<const float4*>(x + i), b = *reinterpret_cast<const float4*>(x + i + 4);
            s = fmaf(a.x, bf16lo_to_f32(p.x), s); s = fmaf(a.y, bf16hi_to_f32(p.x), s);
            s = fmaf(a.z, bf16lo_to_f32(p.y), s); s = fmaf(a.w, bf16hi_to_f32(p.y), s);
            s = fmaf(b.x, bf16lo_to_f32(p.z), s); s = fmaf(b.y, bf16hi_to_f32(p.z), s);
            s = fmaf(b.z, bf16lo_to_f32(p.w), s); s = fmaf(b.w, bf16hi_to_f32(p.w), s);
        }
    } else {
        for (int i = lane; i < n; i += BN_WAVE) s = fmaf(x[i], to_f32(w[i]), s);
    }
    return wave_sum(s);
}

// hidden[pair][f] = act(W_up[e][f] . (w h[t])) for the workgroup's rows f
template <typename T>
__global__ __launch_bounds__(MOE_PAIR_THREADS) void moe_pair_up_kernel(PairArgs a) {
    extern __shared__ __align__(16) float xs[];          // [D]
    const int pair = blockIdx.y, t = pair / a.K;
    const int lane = threadIdx.x & (BN_WAVE - 1), wave = threadIdx.x / BN_WAVE;
    const int e = a.ids[pair];
    if (e >= a.E) return;                                // an identity expert: nothing to multiply
    const float in_scale = a.weight_on_input ? a.wts[pair] : 1.0f;
    const T* h = reinterpret_cast<const T*>(a.h) + (size_t)t * a.ld;
    for (int d = threadIdx.x; d < a.D; d += MOE_PAIR_THREADS) xs[d] = to_f32(from_f32<T>(to_f32(h[d]) * in_scale));
    __syncthreads();
    const T* wu = reinterpret_cast<const T*>(a.w_up) + (size_t)e * (a.gated ? 2 : 1) * a.F * a.D;
    const int f0 = blockIdx.x * MOE_PAIR_ROWS;
    if (a.gated) {
        // a gate row and its up row one after the other, both rows' loads in flight; the products are rounded to the
        // activations' type, as the rows of a stacked product of that type are, before they meet in the unit
        float g[MOE_PAIR_ROWS / (MOE_PAIR_THREADS / BN_WAVE)], u[MOE_PAIR_ROWS / (MOE_PAIR_THREADS / BN_WAVE)];
#pragma unroll
        for (int k = 0; k < MOE_PAIR_ROWS / (MOE_PAIR_THREADS / BN_WAVE); ++k) {
            const int f = f0 + wave + k * (MOE_PAIR_THREADS / BN_WAVE);
            g[k] = f < a.F ? moe_row_dot<T>(wu + (size_t)f * a.D, xs, a.D, lane) : 0.f;
            u[k] = f < a.F ? moe_row_dot<T>(wu + (size_t)(a.F + f) * a.D, xs, a.D, lane) : 0.f;
        }
#pragma unroll
        for (int k = 0; k < MOE_PAIR_ROWS / (MOE_PAIR_THREADS / BN_WAVE); ++k) {
            const int f = f0 + wave + k * (MOE_PAIR_THREADS / BN_WAVE);
            if (f < a.F && lane == 0)
                a.hidden[(size_t)pair * a.F + f] = to_f32(from_f32<T>(moe_clamped_unit(
                    to_f32(from_f32<T>(g[k])), to_f32(from_f32<T>(u[k])), a.limit, a.slope, a.shift)));
        }
        return;
    }
    // a wave's two rows (MOE_PAIR_ROWS / 4) one after the other without a dependence between them: both rows' loads are
    // in flight before the first sum is needed
    float sums[MOE_PAIR_ROWS / (MOE_PAIR_THREADS / BN_WAVE)];
#pragma unroll
    for (int k = 0; k < MOE_PAIR_ROWS / (MOE_PAIR_THREADS / BN_WAVE); ++k) {
        const int f = f0 + wave + k * (MOE_PAIR_THREADS / BN_WAVE);
        sums[k] = f < a.F ? moe_row_dot<T>(wu + (size_t)f * a.D, xs, a.D, lane) : 0.f;
    }
#pragma unroll
    for (int k = 0; k < MOE_PAIR_ROWS / (MOE_PAIR_THREADS / BN_WAVE); ++k) {
        const int f = f0 + wave + k * (MOE_PAIR_THREADS / BN_WAVE);
        if (f < a.F && lane == 0) a.hidden[(size_t)pair * a.F + f] = to_f32(from_f32<T>(bn_unary_act(sums[k], a.act)));
    }
}

// y[j][t][d] = W_down[e][d] . hidden[pair] (times w when the weight multiplies the output) for the workgroup's rows d
template <typename T>
__global__ __launch_bounds__(MOE_PAIR_THREADS) void moe_pair_down_kernel(PairArgs a) {
    extern __shared__ __align__(16) float hid[];         // [F]
    const int pair = blockIdx.y, t = pair / a.K, j = pair - t * a.K;
    const int lane = threadIdx.x & (BN_WAVE - 1), wave = threadIdx.x / BN_WAVE;
    const int e = a.ids[pair];
    const float out_scale = a.weight_on_input ? 1.0f : a.wts[pair];
    if (e >= a.E) {                                      // an identity expert: the token's row times the weight
        const T* h = reinterpret_cast<const T*>(a.h) + (size_t)t * a.ld;
        float* yi = a.y + ((size_t)j * a.T + t) * a.D;
        const int d = blockIdx.x * MOE_PAIR_ROWS + threadIdx.x;
        if (threadIdx.x < MOE_PAIR_ROWS && d < a.D) yi[d] = to_f32(h[d]) * a.wts[pair];
        return;
    }
    for (int f = threadIdx.x; f < a.F; f += MOE_PAIR_THREADS) hid[f] = a.hidden[(size_t)pair * a.F + f];
    __syncthreads();
    const T* wd = reinterpret_cast<const T*>(a.w_down) + (size_t)e * a.D * a.F;
    float* y = a.y + ((size_t)j * a.T + t) * a.D;
    const int d0 = blockIdx.x * MOE_PAIR_ROWS;
    float sums[MOE_PAIR_ROWS / (MOE_PAIR_THREADS / BN_WAVE)];
#pragma unroll
    for (int k = 0; k < MOE_PAIR_ROWS / (MOE_PAIR_THREADS / BN_WAVE); ++k) {
        const int d = d0 + wave + k * (MOE_PAIR_THREADS / BN_WAVE);
        sums[k] = d < a.D ? moe_row_dot<T>(wd + (size_t)d * a.F, hid, a.F, lane) : 0.f;
    }
#pragma unroll
    for (int k = 0; k < MOE_PAIR_ROWS / (MOE_PAIR_THREADS / BN_WAVE); ++k) {
        const int d = d0 + wave + k * (MOE_PAIR_THREADS / BN_WAVE);
        if (d < a.D && lane == 0) y[d] = sums[k] * out_scale;
    }
}

// hidden: float32 work space [n_tokens K, F]; y_rows: the rows of a slab of y (>= n_tokens: the call may take a run of a
// step's tokens, y then points at the run's first row of slab 0)
extern "C" int bn_moe_experts(int dtype, const void* h, int ld, const void* w_up, const void* w_down, const int* ids,
                              const float* wts, float* y, float* hidden, int n_tokens, int y_rows, int D, int F, int E, int K, int act,
                              int weight_on_input, int gated, float limit, float slope, float shift, hipStream_t s) {
    if (n_tokens <= 0 || y_rows < n_tokens || D <= 0 || F <= 0 || E <= 0 || K <= 0 || ld < D) return BN_ERR_ARG;
    if (gated ? !(limit > 0.f) : (act < 0 || act >= BN_UNARY_KINDS)) return BN_ERR_ARG;
    if (!h || !w_up || !w_down || !ids || !wts || !y || !hidden) return BN_ERR_ARG;
    if ((size_t)D * sizeof(float) > 64 * 1024 || (size_t)F * sizeof(float) > 64 * 1024 || (size_t)n_tokens * K > 65535) return BN_ERR_ARG;
    PairArgs a;
    a.h = h; a.w_up = w_up; a.w_down = w_down; a.ids = ids; a.wts = wts; a.y = y; a.hidden = hidden;
    a.ld = ld; a.T = y_rows; a.D = D; a.F = F; a.K = K; a.E = E; a.act = act; a.weight_on_input = weight_on_input ? 1 : 0;
    a.gated = gated ? 1 : 0; a.limit = limit; a.slope = slope; a.shift = shift;
    const dim3 block(MOE_PAIR_THREADS);
    const dim3 up((F + MOE_PAIR_ROWS - 1) / MOE_PAIR_ROWS, n_tokens * K), down((D + MOE_PAIR_ROWS - 1) / MOE_PAIR_ROWS, n_tokens * K);
    if (dtype == BN_DT_F32) {
        hipLaunchKernelGGL(moe_pair_up_kernel<float>, up, block, (size_t)D * sizeof(float), s, a);
        hipLaunchKernelGGL(moe_pair_down_kernel<float>, down, block, (size_t)F * sizeof(float), s, a);
    } else if (dtype == BN_DT_BF16) {
        hipLaunchKernelGGL(moe_pair_up_kernel<bf16>, up, block, (size_t)D * sizeof(float), s, a);
        hipLaunchKernelGGL(moe_pair_down_kernel<bf16>, down, block, (size_t)F * sizeof(float), s, a);
    } else return BN_ERR_DTYPE;
    return bn_launch_status();
}

// ---- steps of many rows: pairs ordered by expert (bf16) ---------------------------------------------------------------
// The pairs of a step are ordered by expert and cut into tiles of up to tile_rows rows of one expert; the inputs are
// gathered in that order (scaled by the pair's weight and rounded, when the weight multiplies the input), and the two
// products run as grouped matrix products over the tiles (gemm_mfma.hip).  Everything a tile needs to know lies in device
// memory, so the launches do not depend on the routing.
#define MOE_PLAN_THREADS 1024

// order [T K]: the pairs (t K + j) by expert, those of identity experts (ids from E on) behind all others and in no tile; tiles [max_tiles][3] = expert, first place in `order`, rows; n_tiles [1]
__global__ __launch_bounds__(MOE_PLAN_THREADS) void moe_plan_kernel(const int* __restrict__ ids, int n_pairs, int E, int tile_rows,
                                                                    int* __restrict__ order, int* __restrict__ tiles,
                                                                    int* __restrict__ n_tiles) {
    __shared__ int count[MOE_MAX_EXPERTS + 1], first[MOE_MAX_EXPERTS + 1], tile0[MOE_MAX_EXPERTS + 1];
    for (int e = threadIdx.x; e <= E; e += blockDim.x) count[e] = 0;
    __syncthreads();
    for (int p = threadIdx.x; p < n_pairs; p += blockDim.x) atomicAdd(&count[min(ids[p], E)], 1);
    __syncthreads();
    if (threadIdx.x == 0) {
        int at = 0, tl = 0;
        for (int e = 0; e < E; ++e) {
            first[e] = at; tile0[e] = tl;
            at += count[e];
            tl += (count[e] + tile_rows - 1) / tile_rows;
        }
        first[E] = at; tile0[E] = tl;
        n_tiles[0] = tl;
    }
    __syncthreads();
    for (int e = threadIdx.x; e < E; e += blockDim.x) {
        const int n = count[e];
        for (int r = 0, k = tile0[e]; r < n; r += tile_rows, ++k) {
            tiles[3 * k] = e; tiles[3 * k + 1] = first[e] + r; tiles[3 * k + 2] = min(tile_rows, n - r);
        }
        count[e] = 0;                                    // now the cursor of the scatter
    }
    if (threadIdx.x == 0) count[E] = 0;
    __syncthreads();
    // the places inside an expert's run are handed out in whatever order the lanes arrive: a row's result does not depend
    // on its place
    for (int p = threadIdx.x; p < n_pairs; p += blockDim.x) {
        const int e = min(ids[p], E);
        order[first[e] + atomicAdd(&count[e], 1)] = p;
    }
}

// xg[place] = h[token of the pair at that place] (times the pair's weight, rounded to bf16, when scale_input); row_map[place]
// = the pair's row of y seen as [K T, D]; row_scale[place] = the pair's weight.  One workgroup a place, 16 bytes a thread.
// The pair of an identity expert (ids from E on) has its result here: its row of y is the token's row times the weight.
__global__ __launch_bounds__(256) void moe_gather_kernel(const bf16* __restrict__ h, int ld, const int* __restrict__ order,
                                                         const float* __restrict__ wts, bf16* __restrict__ xg,
                                                         int* __restrict__ row_map, float* __restrict__ row_scale, int T, int D,
                                                         int K, int scale_input, const int* __restrict__ ids, int E,
                                                         float* __restrict__ y) {
    const int place = blockIdx.x, pair = order[place], t = pair / K, j = pair - t * K;
    const float w = wts[pair];
    if (threadIdx.x == 0) { row_map[place] = j * T + t; row_scale[place] = w; }
    const bf16* src = h + (size_t)t * ld;
    if (ids[pair] >= E) {
        float* yr = y + ((size_t)j * T + t) * D;
        for (int d = 8 * threadIdx.x; d < D; d += 8 * 256) {
            const uint4 p = *reinterpret_cast<const uint4*>(src + d);
            *reinterpret_cast<float4*>(yr + d) = make_float4(bf16lo_to_f32(p.x) * w, bf16hi_to_f32(p.x) * w,
                                                             bf16lo_to_f32(p.y) * w, bf16hi_to_f32(p.y) * w);
            *reinterpret_cast<float4*>(yr + d + 4) = make_float4(bf16lo_to_f32(p.z) * w, bf16hi_to_f32(p.z) * w,
                                                                 bf16lo_to_f32(p.w) * w, bf16hi_to_f32(p.w) * w);
        }
        return;
    }
    bf16* dst = xg + (size_t)place * D;
    for (int d = 8 * threadIdx.x; d < D; d += 8 * 256) {
        uint4 p = *reinterpret_cast<const uint4*>(src + d);
        if (scale_input) {
            uint32_t* q = reinterpret_cast<uint32_t*>(&p);
#pragma unroll
            for (int k = 0; k < 4; ++k) {
                const bf16 lo = __float2bfloat16(bf16lo_to_f32(q[k]) * w), hi = __float2bfloat16(bf16hi_to_f32(q[k]) * w);
                q[k] = (uint32_t)__builtin_bit_cast(unsigned short, lo) | ((uint32_t)__builtin_bit_cast(unsigned short, hi) << 16);
            }
        }
        *reinterpret_cast<uint4*>(dst + d) = p;
    }
}

extern "C" int bn_moe_grouped_tiles(int n_pairs, int E, int tile_rows) {
    return tile_rows > 0 ? (n_pairs + tile_rows - 1) / tile_rows + E : 0;
}

// y: float32 [K, n_tokens, D], of which the identity experts' rows are written here
// work: int32 [2 n_pairs + 3 max_tiles + 1] = order, row_map, tiles, n_tiles; row_scale: float32 [n_pairs]; xg: bf16 [n_pairs, D]
extern "C" int bn_moe_group(const void* h, int ld, const int* ids, const float* wts, int* work, float* row_scale, void* xg,
                            int n_tokens, int D, int E, int K, int tile_rows, int scale_input, float* y, hipStream_t s) {
    if (n_tokens <= 0 || K <= 0 || E <= 0 || E > MOE_MAX_EXPERTS || D <= 0 || D % 8 || ld < D || ld % 8 || tile_rows <= 0) return BN_ERR_ARG;
    if (!h || !ids || !wts || !work || !row_scale || !xg || !y || (((uintptr_t)h | (uintptr_t)xg | (uintptr_t)y) & 15)) return BN_ERR_ARG;
    const int n_pairs = n_tokens * K, max_tiles = bn_moe_grouped_tiles(n_pairs, E, tile_rows);
    int* order = work;
    int* row_map = work + n_pairs;
    int* tiles = row_map + n_pairs;
    int* n_tiles = tiles + 3 * max_tiles;
    hipLaunchKernelGGL(moe_plan_kernel, dim3(1), dim3(MOE_PLAN_THREADS), 0, s, ids, n_pairs, E, tile_rows, order, tiles, n_tiles);
    hipLaunchKernelGGL(moe_gather_kernel, dim3(n_pairs), dim3(256), 0, s, (const bf16*)h, ld, order, wts, (bf16*)xg, row_map,
                       row_scale, n_tokens, D, K, scale_input ? 1 : 0, ids, E, y);
    return bn_launch_status();
}

// ---- the clamped gated unit over rows of stacked products ------------------------------------------------------------
// out[r, f] = unit(gu[r, f], gu[r, F + f]) (times row_scale[r]), rounded once to the activations' type: what follows a
// product with stacked gate and up rows, for the grouped experts and for a shared expert (whose factor is its gate)
template <typename T>
__global__ void gated_unit_kernel(T* __restrict__ out, const T* __restrict__ gu, int ld, const float* __restrict__ row_scale,
                                  int n_rows, int F, float limit, float slope, float shift) {
    const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= (size_t)n_rows * F) return;
    const int r = (int)(i / F), f = (int)(i - (size_t)r * F);
    const T* row = gu + (size_t)r * ld;
    float v = moe_clamped_unit(to_f32(row[f]), to_f32(row[F + f]), limit, slope, shift);
    if (row_scale) v *= row_scale[r];
    out[i] = from_f32<T>(v);
}

// the same for bf16 rows of whole 16-byte groups: a thread takes eight consecutive columns
__global__ __launch_bounds__(256) void gated_unit_bf16x8_kernel(bf16* __restrict__ out, const bf16* __restrict__ gu, int ld,
                                                                const float* __restrict__ row_scale, int F, float limit, float slope,
                                                                float shift) {
    const int r = blockIdx.y, f = 8 * (blockIdx.x * 256 + threadIdx.x);
    if (f >= F) return;
    const bf16* row = gu + (size_t)r * ld;
    const uint4 g = *reinterpret_cast<const uint4*>(row + f), u = *reinterpret_cast<const uint4*>(row + F + f);
    const uint32_t gw[4] = {g.x, g.y, g.z, g.w}, uw[4] = {u.x, u.y, u.z, u.w};
    const float s = row_scale ? row_scale[r] : 1.0f;
    bf16 o[8];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
        float a = moe_clamped_unit(bf16lo_to_f32(gw[k]), bf16lo_to_f32(uw[k]), limit, slope, shift);
        float b = moe_clamped_unit(bf16hi_to_f32(gw[k]), bf16hi_to_f32(uw[k]), limit, slope, shift);
        if (row_scale) { a *= s; b *= s; }
        o[2 * k] = from_f32<bf16>(a);
        o[2 * k + 1] = from_f32<bf16>(b);
    }
    *reinterpret_cast<uint4*>(out + (size_t)r * F + f) = *reinterpret_cast<const uint4*>(o);
}

extern "C" int bn_gated_unit(int dtype, void* out, const void* gu, int ld, const float* row_scale, int n_rows, int F, float limit,
                             float slope, float shift, hipStream_t s) {
    if (n_rows <= 0 || F <= 0 || ld < 2 * F || !out || !gu || !(limit > 0.f)) return BN_ERR_ARG;
    const size_t n = (size_t)n_rows * F;
    const dim3 grid((unsigned)((n + 255) / 256)), block(256);
    if (dtype == BN_DT_BF16 && F % 8 == 0 && ld % 8 == 0 && n_rows <= 65535 && !(((uintptr_t)out | (uintptr_t)gu) & 15)) {
        hipLaunchKernelGGL(gated_unit_bf16x8_kernel, dim3((F + 2047) / 2048, n_rows), block, 0, s, (bf16*)out, (const bf16*)gu, ld,
                           row_scale, F, limit, slope, shift);
        return bn_launch_status();
    }
    if (dtype == BN_DT_F32)
        hipLaunchKernelGGL(gated_unit_kernel<float>, grid, block, 0, s, (float*)out, (const float*)gu, ld, row_scale, n_rows, F, limit, slope, shift);
    else if (dtype == BN_DT_BF16)
        hipLaunchKernelGGL(gated_unit_kernel<bf16>, grid, block, 0, s, (bf16*)out, (const bf16*)gu, ld, row_scale, n_rows, F, limit, slope, shift);
    else return BN_ERR_DTYPE;
    return bn_launch_status();
}
