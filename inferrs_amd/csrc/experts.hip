// Routed experts: a router scores every expert for a token, the `top` best are run and their outputs added up
// with the scores as weights.
//
//   route      a wave a token: router logits as 32-bit sums whatever row and matrix are stored in, scores = sigmoid
//              (or softmax), the top experts by score (ties: the lower index), weights = score * scale (optionally
//              renormalised over the chosen).
//   plan       one block: the (token, k) pairs ordered by expert, and a table of row tiles (expert, first pair, rows),
//              all on the device: the host never learns how many tokens an expert got.
//   gate_up    tile by tile: rows gathered by pair, act(gate, up) in the epilogue.
//   down       tile by tile: one 32-bit output row a pair; whoever adds the experts up takes the pairs of a token
//              in the order of k, so a token's sum does not depend on what else is in the batch.
#include "api.h"
#include "common.h"
#include "tile_fma.h"
#include "tile_mfma.h"

#define IA_MAX_EXPERTS 256
#define IA_MAX_TOP 16

enum { IA_SCORE_SIGMOID = 0, IA_SCORE_SOFTMAX = 1 };

// eight neighbouring values of a row as 32-bit floats
__device__ __forceinline__ void load8(const float* p, float (&v)[8]) {
    const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
    v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
}
__device__ __forceinline__ void load8(const bf16_t* p, float (&v)[8]) {
    const uint4 a = *reinterpret_cast<const uint4*>(p);
    const uint32_t w[4] = {a.x, a.y, a.z, a.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        v[2 * i] = __uint_as_float(w[i] << 16);
        v[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
    }
}

// One wave: a token's choice and weights from its logits (of E rows of the router's matrix, the last `gates` of which take no
// part in it).  Q: registers of logits a lane (E - gates up to 64 Q).
template <int Q>
__device__ __forceinline__ void route_pick(int* __restrict__ sel, float* __restrict__ weight, const float* logits, int t, int lane, int E,
                                           int top, float scale, int score_fn, int renorm, const float* __restrict__ choice_bias,
                                           int gates, float* __restrict__ gate_out, int group_count, int group_keep,
                                           int* chosen = nullptr) {
    if (gates > 0) {
        E -= gates;
        for (int j = lane; j < gates; j += IA_WAVE) gate_out[(long long)t * gates + j] = 1.0f / (1.0f + expf(-logits[E + j]));
    }
    float z[Q];             // expert e lives in lane e % 64, register e / 64
#pragma unroll
    for (int q = 0; q < Q; ++q) {
        const int e = q * IA_WAVE + lane;
        z[q] = e < E ? logits[e] : -INFINITY;
    }
    float zmax = -INFINITY, denom = 1.f;
    if (score_fn == IA_SCORE_SOFTMAX) {
#pragma unroll
        for (int q = 0; q < Q; ++q) zmax = fmaxf(zmax, z[q]);
        zmax = wave_max(zmax);
        float s = 0.f;
#pragma unroll
        for (int q = 0; q < Q; ++q) s += z[q] > -INFINITY ? expf(z[q] - zmax) : 0.f;
        denom = wave_sum(s);
    }
    auto score = [&](float x) { return score_fn == IA_SCORE_SOFTMAX ? expf(x - zmax) / denom : 1.0f / (1.0f + expf(-x)); };
    if (group_count > 1) {
        // The outputs form `group_count` groups of neighbours; a group is worth the sum of its two largest scores (with the
        // choice's bias), and only outputs of the `group_keep` best groups stay in the choice (of equal groups the lower).
        const int size = E / group_count;
        float worth[Q];     // group g lives in lane g % 64, register g / 64
#pragma unroll
        for (int q = 0; q < Q; ++q) {
            const int g = q * IA_WAVE + lane;
            float one = -INFINITY, two = -INFINITY;
            for (int i = 0; g < group_count && i < size; ++i) {
                const int e = g * size + i;
                const float s = score(logits[e]) + (choice_bias != nullptr ? choice_bias[e] : 0.f);
                if (s > one) { two = one; one = s; }
                else if (s > two) two = s;
            }
            worth[q] = g < group_count ? one + (size > 1 ? two : 0.f) : -INFINITY;
        }
        int in = 0;         // bit q: the group in register q stays
        for (int k = 0; k < group_keep; ++k) {
            float best = -INFINITY;
            int best_g = 0x7fffffff;
#pragma unroll
            for (int q = 0; q < Q; ++q)
                if (!((in >> q) & 1) && worth[q] > best) { best = worth[q]; best_g = q * IA_WAVE + lane; }
#pragma unroll
            for (int o = IA_WAVE / 2; o > 0; o >>= 1) {
                const float ob = __shfl_xor(best, o, IA_WAVE);
                const int og = __shfl_xor(best_g, o, IA_WAVE);
                if (ob > best || (ob == best && og < best_g)) { best = ob; best_g = og; }
            }
            if (best_g % IA_WAVE == lane) in |= 1 << (best_g / IA_WAVE);
        }
#pragma unroll
        for (int q = 0; q < Q; ++q) {
            const int e = q * IA_WAVE + lane, g = e < E ? e / size : 0;
            const int kept = __shfl(in, g % IA_WAVE, IA_WAVE);
            if (!((kept >> (g / IA_WAVE)) & 1)) z[q] = -INFINITY;
        }
    }
    float total = 0.f, mine = 0.f;
    int mine_e = 0;
    if (choice_bias != nullptr) {
        // The choice goes by score + bias, the weights by the score alone: the scores are formed first, and the picking
        // walks the biased ones (of equal ones the lower index).
        float sc[Q], key[Q];
#pragma unroll
        for (int q = 0; q < Q; ++q) {
            const int e = q * IA_WAVE + lane;
            sc[q] = e < E ? score(z[q]) : 0.f;
            key[q] = e < E && z[q] > -INFINITY ? sc[q] + choice_bias[e] : -INFINITY;
        }
        for (int k = 0; k < top; ++k) {
            float best = -INFINITY, best_s = 0.f;
            int best_e = 0x7fffffff;
#pragma unroll
            for (int q = 0; q < Q; ++q)
                if (key[q] > best) { best = key[q]; best_e = q * IA_WAVE + lane; best_s = sc[q]; }
#pragma unroll
            for (int o = IA_WAVE / 2; o > 0; o >>= 1) {
                const float ob = __shfl_xor(best, o, IA_WAVE), os = __shfl_xor(best_s, o, IA_WAVE);
                const int oe = __shfl_xor(best_e, o, IA_WAVE);
                if (ob > best || (ob == best && oe < best_e)) { best = ob; best_e = oe; best_s = os; }
            }
#pragma unroll
            for (int q = 0; q < Q; ++q)
                if (best_e == q * IA_WAVE + lane) key[q] = -INFINITY;
            total += best_s;
            if (lane == k) { mine = best_s; mine_e = best_e; }
        }
    } else
    for (int k = 0; k < top; ++k) {
        // every lane's best, then the wave's: the largest logit, of equal ones the lower index
        float best = -INFINITY;
        int best_e = 0x7fffffff;
#pragma unroll
        for (int q = 0; q < Q; ++q)
            if (z[q] > best) { best = z[q]; best_e = q * IA_WAVE + lane; }
#pragma unroll
        for (int o = IA_WAVE / 2; o > 0; o >>= 1) {
            const float ob = __shfl_xor(best, o, IA_WAVE);
            const int oe = __shfl_xor(best_e, o, IA_WAVE);
            if (ob > best || (ob == best && oe < best_e)) { best = ob; best_e = oe; }
        }
#pragma unroll
        for (int q = 0; q < Q; ++q)
            if (best_e == q * IA_WAVE + lane) z[q] = -INFINITY;
        const float s = score(best);
        total += s;
        if (lane == k) { mine = s; mine_e = best_e; }
    }
    if (lane < top) {
        sel[(long long)t * top + lane] = mine_e;
        if (chosen != nullptr) chosen[lane] = mine_e;
        weight[(long long)t * top + lane] = (renorm ? mine / (total + 1e-20f) : mine) * scale;     // (scores that are all zero stay zero)
    }
}

#define IA_ROUTE_WAVES 4        // waves of a token's block
#define IA_ROUTE_FEW_TOKENS 64 // up to this many tokens a step the blocks are too few to hide a wave's chain of loads
#define IA_ROUTE_SHARE 8        // experts whose sums a wave holds at a time: a block takes 32 experts a round (routers of 33 to 64
                                // outputs: 10, 12 or 16, so that one walk over the row serves them all)

// The logits: a block of four waves a token; in every round of 32 experts a wave takes eight.  A lane owns the features
// 8 lane + 512 i of the row and adds its products up in that order (32-bit multiply-adds), then the lanes' sums meet in a
// butterfly: an order that depends on the width alone.  The logits meet in shared memory and the first wave picks.
// VEC: the width is a multiple of 8 (16-byte loads); else element by element.
// WAVES: the block's waves.  A logit is one wave's walk over the row whatever SHARE and WAVES are, so neither changes a sum.
template <typename T, bool VEC, int SHARE = IA_ROUTE_SHARE, int WAVES = IA_ROUTE_WAVES>
__global__ __launch_bounds__(64 * WAVES) void route_kernel(int* __restrict__ sel, float* __restrict__ weight,
                                                                    const T* __restrict__ h, const T* __restrict__ wr, int n,
                                                                    int W, int E, int top, float scale, int score_fn,
                                                                    int renorm, const float* __restrict__ choice_bias,
                                                                    int gates, float* __restrict__ gate_out, int group_count, int group_keep) {
    // E counts every row of the router's matrix: the last `gates` of them take no part in the choice; the sigmoid of
    // such a row's logit is handed out as it is (gate_out [n, gates]): a gate a token, formed like a router's logit.
    __shared__ float logits[IA_MAX_EXPERTS];
    const int t = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const T* row = h + (long long)t * W;
    for (int e0 = wave * SHARE; e0 < E; e0 += WAVES * SHARE) {
        float acc[SHARE];
#pragma unroll
        for (int j = 0; j < SHARE; ++j) acc[j] = 0.f;
        // (four rounds of loads under way at once: a round is a trip to the memory)
#pragma unroll 4
        for (int c0 = lane * 8; c0 < W; c0 += IA_WAVE * 8) {
            float x[8];
            if (VEC) {
                load8(row + c0, x);
            } else {
#pragma unroll
                for (int i = 0; i < 8; ++i) x[i] = c0 + i < W ? ld(row + c0 + i) : 0.f;
            }
#pragma unroll
            for (int j = 0; j < SHARE; ++j) {
                // (an expert beyond the last reads the last one's row: no branch stands between the loads)
                const T* w = wr + (long long)(e0 + j < E ? e0 + j : E - 1) * W + c0;
                float wv[8];
                if (VEC) {
                    load8(w, wv);
                } else {
#pragma unroll
                    for (int i = 0; i < 8; ++i) wv[i] = c0 + i < W ? ld(w + i) : 0.f;
                }
#pragma unroll
                for (int i = 0; i < 8; ++i) acc[j] = fmaf(x[i], wv[i], acc[j]);
            }
        }
#pragma unroll
        for (int j = 0; j < SHARE; ++j) {
            const float total = wave_sum(acc[j]);
            if (lane == 0 && e0 + j < E) logits[e0 + j] = total;
        }
    }
    __syncthreads();
    if (wave != 0) return;
    route_pick<IA_MAX_EXPERTS / IA_WAVE>(sel, weight, logits, t, lane, E, top, scale, score_fn, renorm, choice_bias, gates, gate_out, group_count, group_keep);
}

// The whole block.  `order` [pairs]: the pairs grouped by expert; tiles: expert, first place in `order`, rows; meta[0]: tiles.
// sel may lie in shared memory.
struct RoutePlan {
    int *order, *tile_expert, *tile_first, *tile_rows, *meta;
    int E, tile;                                   // experts with weights, rows of a tile; order null: no plan
};
__device__ __forceinline__ void route_plan_block(const RoutePlan& p, const int* sel, int pairs) {
    int *order = p.order, *tile_expert = p.tile_expert, *tile_first = p.tile_first, *tile_rows = p.tile_rows, *meta = p.meta;
    const int E = p.E, tile = p.tile;
    __shared__ int count[IA_MAX_EXPERTS], first[IA_MAX_EXPERTS], tile0[IA_MAX_EXPERTS], cursor[IA_MAX_EXPERTS];
    for (int e = threadIdx.x; e < E; e += blockDim.x) count[e] = cursor[e] = 0;
    __syncthreads();
    // (a choice of E or beyond names no expert with weights: such a pair gets no place and no tile)
    for (int p = threadIdx.x; p < pairs; p += blockDim.x)
        if (sel[p] < E) atomicAdd(&count[sel[p]], 1);
    __syncthreads();
    if (threadIdx.x < IA_WAVE) {                   // (running sums over the experts, 64 at a time by lane shifts)
        int at = 0, tiles = 0;
        for (int e0 = 0; e0 < E; e0 += IA_WAVE) {
            const int e = e0 + (int)threadIdx.x;
            const int mine = e < E ? count[e] : 0, mine_t = (mine + tile - 1) / tile;
            int sum = mine, sum_t = mine_t;
#pragma unroll
            for (int o = 1; o < IA_WAVE; o <<= 1) {
                const int u = __shfl_up(sum, o, IA_WAVE), v = __shfl_up(sum_t, o, IA_WAVE);
                if ((int)threadIdx.x >= o) { sum += u; sum_t += v; }
            }
            if (e < E) { first[e] = at + sum - mine; tile0[e] = tiles + sum_t - mine_t; }
            at += __shfl(sum, IA_WAVE - 1, IA_WAVE);
            tiles += __shfl(sum_t, IA_WAVE - 1, IA_WAVE);
        }
        if (threadIdx.x == 0) meta[0] = tiles;
    }
    __syncthreads();
    for (int e = threadIdx.x; e < E; e += blockDim.x) {
        const int tiles = (count[e] + tile - 1) / tile;
        for (int i = 0; i < tiles; ++i) {
            tile_expert[tile0[e] + i] = e;
            tile_first[tile0[e] + i] = first[e] + i * tile;
            tile_rows[tile0[e] + i] = min(tile, count[e] - i * tile);
        }
    }
    for (int p = threadIdx.x; p < pairs; p += blockDim.x) {
        const int e = sel[p];
        if (e < E) order[first[e] + atomicAdd(&cursor[e], 1)] = p;
    }
}

__global__ __launch_bounds__(1024) void route_plan_kernel(const RoutePlan p, const int* __restrict__ sel, int pairs) {
    route_plan_block(p, sel, pairs);
}

// The router on the matrix cores, for bfloat16 rows and matrices (every product exact, the sums 32-bit) of up to 64 outputs: a
// block of sixteen waves owns 16 tokens; wave w multiplies the steps w, w + 16, .. of 32 features, the waves' sums meet in
// shared memory and are added in the waves' order (an order that depends on the width alone), then wave w picks for token
// w.  A step of up to 16 tokens is one block, which then orders the pairs for the experts' products as well (`plan`): one
// kernel where there were two.
#define IA_RM_WAVES 16
#define IA_RM_TOKENS 16
template <int NT>
__global__ __launch_bounds__(64 * IA_RM_WAVES) void route_mfma_kernel(int* __restrict__ sel, float* __restrict__ weight,
                                                                      const bf16_t* __restrict__ h, const bf16_t* __restrict__ wr, int n,
                                                                      int W, int E, int top, float scale, int score_fn, int renorm,
                                                                      const float* __restrict__ choice_bias, int gates,
                                                                      float* __restrict__ gate_out, int group_count, int group_keep, const RoutePlan plan) {
    extern __shared__ float rm_part[];             // [waves][tokens][16 NT]
    __shared__ float logits[IA_RM_TOKENS][16 * NT];
    __shared__ int chosen[IA_RM_TOKENS * IA_MAX_TOP];
    const int t0 = blockIdx.x * IA_RM_TOKENS, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int r16 = lane & 15, G = lane >> 4;
    const bf16_t* row = h + (long long)(t0 + r16 < n ? t0 + r16 : n - 1) * W;
    const bf16_t* w[NT];
#pragma unroll
    for (int j = 0; j < NT; ++j) w[j] = wr + (long long)(16 * j + r16 < E ? 16 * j + r16 : E - 1) * W;
    tm_f32x4 acc[NT];
#pragma unroll
    for (int j = 0; j < NT; ++j) acc[j] = (tm_f32x4){0.f, 0.f, 0.f, 0.f};
    const int steps = (W + 31) / 32;
#pragma unroll 4
    for (int st = wave; st < steps; st += IA_RM_WAVES) {
        const int c = 32 * st + 8 * G;
        const bool in = c < W;                     // (widths in steps of 8: a piece lies inside or outside as a whole)
        const tm_u32x4 zero = {0u, 0u, 0u, 0u};
        const tm_u32x4 x = in ? *reinterpret_cast<const tm_u32x4*>(row + c) : zero;
#pragma unroll
        for (int j = 0; j < NT; ++j) {
            const tm_u32x4 b = in ? *reinterpret_cast<const tm_u32x4*>(w[j] + c) : zero;
            acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(tm_bf16x8, x), __builtin_bit_cast(tm_bf16x8, b), acc[j], 0, 0, 0);
        }
    }
#pragma unroll
    for (int j = 0; j < NT; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) rm_part[(wave * IA_RM_TOKENS + 4 * G + i) * 16 * NT + 16 * j + r16] = acc[j][i];
    __syncthreads();
    if (threadIdx.x < IA_RM_TOKENS * 16 * NT) {
        float total = 0.f;
#pragma unroll
        for (int q = 0; q < IA_RM_WAVES; ++q) total += rm_part[q * IA_RM_TOKENS * 16 * NT + threadIdx.x];
        (&logits[0][0])[threadIdx.x] = total;
    }
    __syncthreads();
    if (t0 + wave < n)
        route_pick<1>(sel, weight, logits[wave], t0 + wave, lane, E, top, scale, score_fn, renorm, choice_bias, gates, gate_out, group_count, group_keep,
                      chosen + wave * top);
    if (plan.order == nullptr) return;             // (the same for all threads; the grid is one block otherwise)
    __syncthreads();
    route_plan_block(plan, chosen, n * top);
}

// The choice from logits that another product has left in 32-bit rows, for steps of up to 16 tokens: a wave a token, then the
// plan.  (A router's matrix read by one compute unit takes as long as the unit's share of the memory's rate lets it; as rows
// of a large product beside it, it is spread over the chip.)
__global__ __launch_bounds__(64 * IA_RM_WAVES) void route_logits_kernel(int* __restrict__ sel, float* __restrict__ weight,
                                                                        const float* __restrict__ logits, long long ld, int n, int E,
                                                                        int top, float scale, int score_fn, int renorm,
                                                                        const float* __restrict__ choice_bias, int gates,
                                                                        float* __restrict__ gate_out, int group_count, int group_keep, const RoutePlan plan) {
    __shared__ int chosen[IA_RM_TOKENS * IA_MAX_TOP];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    if (wave < n) {
        if (E - gates <= IA_WAVE)
            route_pick<1>(sel, weight, logits + wave * ld, wave, lane, E, top, scale, score_fn, renorm, choice_bias, gates, gate_out, group_count, group_keep,
                          chosen + wave * top);
        else
            route_pick<IA_MAX_EXPERTS / IA_WAVE>(sel, weight, logits + wave * ld, wave, lane, E, top, scale, score_fn, renorm, choice_bias,
                                                 gates, gate_out, group_count, group_keep, chosen + wave * top);
    }
    __syncthreads();
    route_plan_block(plan, chosen, n * top);
}

// An expert's activation over its two sums.  Clamped: g' * sigmoid(alpha g') * (u' + 1), g' = min(g, limit), u' = clamp(u,
// -limit, limit); plain (IA_EXPERT_SILU): silu(g) * u.  The choice is the same for all lanes of a launch.
enum { IA_EXPERT_CLAMPED = 0, IA_EXPERT_SILU = 1 };
__device__ __forceinline__ float expert_act(float g, float u, float limit, float alpha, int form) {
    if (form == IA_EXPERT_SILU) return g / (1.0f + expf(-g)) * u;
    const float gv = fminf(g, limit), uv = fminf(fmaxf(u, -limit), limit);
    return gv / (1.0f + expf(-alpha * gv)) * (uv + 1.0f);
}

// act[place][j] = expert_act(gate_j . x, up_j . x);
// x = h[pair / top] (times in_weight[pair], where given: 32-bit, one a pair).  w_gu [E][2 ff][W]: an expert's gate rows, then its up rows.
template <typename T>
__global__ __launch_bounds__(256) void experts_gate_up_kernel(T* __restrict__ act, const T* __restrict__ h,
                                                              const T* __restrict__ w_gu, const int* __restrict__ order,
                                                              const int* __restrict__ tile_expert,
                                                              const int* __restrict__ tile_first,
                                                              const int* __restrict__ tile_rows,
                                                              const int* __restrict__ meta, int top, int W, int ff,
                                                              float limit, float alpha, int form,
                                                              const float* __restrict__ in_weight) {
    __shared__ TileShared sh;
    const int tile = blockIdx.y;
    if (tile >= meta[0]) return;
    const int e = tile_expert[tile], first = tile_first[tile], rows = tile_rows[tile], col0 = blockIdx.x * IA_TN;
    float g[2][4], u[2][4];
    auto xrow = [&](int i) -> const T* { return i < rows ? h + (long long)(order[first + i] / top) * W : nullptr; };
    const T* wg = w_gu + ((long long)e * 2 * ff + col0) * W;
    tile_product<T, T, true>(g, u, sh, xrow, wg, wg + (long long)ff * W, ff - col0, W, W);
    const int ty = threadIdx.x >> 4, tx = threadIdx.x & 15;
#pragma unroll
    for (int a = 0; a < 2; ++a) {
        const int i = 2 * ty + a;
        if (i >= rows) continue;
        // (in_weight: the pair's weight is a factor on the expert's INPUT, hence on both sums ahead of the limits)
        const float wi = in_weight != nullptr ? in_weight[order[first + i]] : 1.0f;
#pragma unroll
        for (int b = 0; b < 4; ++b) {
            const int j = col0 + 4 * tx + b;
            if (j >= ff) continue;
            st(act + (long long)(first + i) * ff + j, expert_act(g[a][b] * wi, u[a][b] * wi, limit, alpha, form));
        }
    }
}

// y[pair][c] = down_c . act[place]   (32-bit rows, one a pair)
template <typename T>
__global__ __launch_bounds__(256) void experts_down_kernel(float* __restrict__ y, const T* __restrict__ act,
                                                           const T* __restrict__ w_down, const int* __restrict__ order,
                                                           const int* __restrict__ tile_expert,
                                                           const int* __restrict__ tile_first,
                                                           const int* __restrict__ tile_rows,
                                                           const int* __restrict__ meta, int W, int ff) {
    __shared__ TileShared sh;
    const int tile = blockIdx.y;
    if (tile >= meta[0]) return;
    const int e = tile_expert[tile], first = tile_first[tile], rows = tile_rows[tile], col0 = blockIdx.x * IA_TN;
    float acc[2][4], unused[2][4];
    auto xrow = [&](int i) -> const T* { return i < rows ? act + (long long)(first + i) * ff : nullptr; };
    const T* wd = w_down + ((long long)e * W + col0) * ff;
    tile_product<T, T, false>(acc, unused, sh, xrow, wd, wd, W - col0, ff, ff);
    const int ty = threadIdx.x >> 4, tx = threadIdx.x & 15;
#pragma unroll
    for (int a = 0; a < 2; ++a) {
        const int i = 2 * ty + a;
        if (i >= rows) continue;
        const long long pair = order[first + i];
#pragma unroll
        for (int b = 0; b < 4; ++b) {
            const int c = col0 + 4 * tx + b;
            if (c < W) y[pair * W + c] = acc[a][b];
        }
    }
}

// The same two products on the matrix cores (bfloat16; widths in steps of 8) over weights stored as tiles (see
// tile_mfma.h): w_gu [E][2][ceil(ff / 64)][ceil(W / 64)][64][64], w_down [E][ceil(W / 64)][ceil(ff / 64)][64][64].
template <int RT, int FT>
__global__ __launch_bounds__(256) void experts_gate_up_mfma_kernel(bf16_t* __restrict__ act, const bf16_t* __restrict__ h,
                                                                   const bf16_t* __restrict__ w_gu,
                                                                   const int* __restrict__ order,
                                                                   const int* __restrict__ tile_expert,
                                                                   const int* __restrict__ tile_first,
                                                                   const int* __restrict__ tile_rows,
                                                                   const int* __restrict__ meta, int top, int W, int ff,
                                                                   float limit, float alpha, int form,
                                                              const float* __restrict__ in_weight) {
    using Tile = TileMfma<RT, FT, 64, true>;
    __shared__ typename Tile::Shared sh;
    const int tile = blockIdx.y;
    if (tile >= meta[0]) return;
    const int e = tile_expert[tile], first = tile_first[tile], rows = tile_rows[tile], col0 = blockIdx.x * Tile::FEATURES;
    const int fbs = (ff + 63) / 64, chunks = (W + 63) / 64;
    tm_f32x4 g[FT][RT], u[FT][RT];
    auto xrow = [&](int i) -> const bf16_t* { return i < rows ? h + (long long)(order[first + i] / top) * W : nullptr; };
    const long long matrix = (long long)fbs * chunks * 4096;
    const bf16_t* wg = w_gu + (long long)e * 2 * matrix + (long long)(col0 / 64) * chunks * 4096;
    Tile::product_tiled(g, u, sh, xrow, wg, wg + matrix, fbs - col0 / 64, chunks, W);
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
        const int i = 16 * rt + (lane & 15);
        const float wi = in_weight != nullptr && i < rows ? in_weight[order[first + i]] : 1.0f;
#pragma unroll
        for (int ft = 0; ft < FT; ++ft) {
            const int j0 = col0 + 16 * (wave * FT + ft) + 4 * (lane >> 4);
            const tm_f32x4 gq = g[ft][rt], uq = u[ft][rt];
            const float gs[4] = {gq[0], gq[1], gq[2], gq[3]}, us[4] = {uq[0], uq[1], uq[2], uq[3]};
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                if (i >= rows || j0 + q >= ff) continue;
                st(act + (long long)(first + i) * ff + j0 + q, expert_act(gs[q] * wi, us[q] * wi, limit, alpha, form));
            }
        }
    }
}

template <int RT, int FT>
__global__ __launch_bounds__(256) void experts_down_mfma_kernel(float* __restrict__ y, const bf16_t* __restrict__ act,
                                                                const bf16_t* __restrict__ w_down,
                                                                const int* __restrict__ order,
                                                                const int* __restrict__ tile_expert,
                                                                const int* __restrict__ tile_first,
                                                                const int* __restrict__ tile_rows,
                                                                const int* __restrict__ meta, int W, int ff) {
    using Tile = TileMfma<RT, FT, 64, false>;
    __shared__ typename Tile::Shared sh;
    const int tile = blockIdx.y;
    if (tile >= meta[0]) return;
    const int e = tile_expert[tile], first = tile_first[tile], rows = tile_rows[tile], col0 = blockIdx.x * Tile::FEATURES;
    const int fbs = (W + 63) / 64, chunks = (ff + 63) / 64;
    tm_f32x4 acc[FT][RT], unused[FT][RT];
    auto xrow = [&](int i) -> const bf16_t* { return i < rows ? act + (long long)(first + i) * ff : nullptr; };
    const bf16_t* wd = w_down + ((long long)e * fbs + col0 / 64) * chunks * 4096;
    Tile::product_tiled(acc, unused, sh, xrow, wd, wd, fbs - col0 / 64, chunks, ff);
    Tile::each([&](int i, int f, int ft, int rt, int q) {
        const int c = col0 + f;
        if (i < rows && c < W) y[(long long)order[first + i] * W + c] = acc[ft][rt][q];
    });
}

static bool route_mfma_fits(int W, int rows, int dtype, const void* h, const void* router) {
    return dtype == IA_BF16 && rows <= 64 && W % 8 == 0 && W >= 128 && tile_mfma_aligned(h) && tile_mfma_aligned(router);
}
// Whether `ia_route` makes the plan of this step itself (rows: every row of the router's matrix).
extern "C" int ia_route_plans(int n, int W, int rows, int dtype, const void* h, const void* router) {
    return n <= IA_RM_TOKENS && route_mfma_fits(W, rows, dtype, h, router) ? 1 : 0;
}

// group_count 0 or 1: no groups; else the outputs form that many equal groups of neighbours, of which the group_keep best (by
// the sum of their two largest scores) stay in the choice.
static bool route_groups_fit(int E, int top, int group_count, int group_keep) {
    return group_count <= 1 || (E % group_count == 0 && group_keep >= 1 && group_keep <= group_count && top <= group_keep * (E / group_count));
}

// choice_bias: null, or [E] 32-bit values added to the scores for the choice only (the weights are the scores themselves)
extern "C" int ia_route(int* sel, float* weight, const void* h, const void* router, int n, int W, int E, int top,
                        float scale, int score_fn, int renorm, const float* choice_bias, int gates, float* gate_out,
                        int group_count, int group_keep, int* order, int* tile_expert, int* tile_first, int* tile_rows,
                        int* meta, int plan_E, int tile, int dtype, hipStream_t stream) {
    // order: null, or the plan of `ia_route_plan` is made as well (ia_route_plans(...) says for which steps)
    // E: the router's outputs that can be chosen; the matrix holds `gates` more rows behind them (see the kernel)
    IA_CHECK(gates >= 0 && (gates == 0 || gate_out != nullptr), "route: %d gate rows need a place for their values", gates);
    IA_CHECK(n >= 0 && W > 0 && E >= 1 && E + gates <= IA_MAX_EXPERTS && top >= 1 && top <= E && top <= IA_MAX_TOP,
             "route: n=%d width=%d experts=%d and %d gate rows (up to %d) top=%d (up to %d)", n, W, E, gates, IA_MAX_EXPERTS, top, IA_MAX_TOP);
    IA_CHECK(route_groups_fit(E, top, group_count, group_keep), "route: %d of %d groups of %d outputs, top %d", group_keep, group_count, E, top);
    E += gates;
    IA_CHECK(score_fn == IA_SCORE_SIGMOID || score_fn == IA_SCORE_SOFTMAX, "route: unknown score function %d", score_fn);
    IA_CHECK(order == nullptr || ia_route_plans(n, W, E, dtype, h, router), "route: this step's plan is made by a kernel of its own");
    if (n == 0) return 0;
    if (route_mfma_fits(W, E, dtype, h, router)) {
        RoutePlan plan;
        plan.order = order; plan.tile_expert = tile_expert; plan.tile_first = tile_first; plan.tile_rows = tile_rows; plan.meta = meta;
        plan.E = plan_E; plan.tile = tile;
        const int nt = (E + 15) / 16;
        const unsigned blocks = (unsigned)((n + IA_RM_TOKENS - 1) / IA_RM_TOKENS);
        const size_t shm = (size_t)IA_RM_WAVES * IA_RM_TOKENS * 16 * nt * sizeof(float);
#define IA_RM(NT)                                                                                                       \
    do {                                                                                                                \
        static int asked = 0;                                                                                           \
        if (shm > 48 * 1024 && !asked) {                                                                                \
            const hipError_t e = hipFuncSetAttribute((const void*)route_mfma_kernel<NT>, hipFuncAttributeMaxDynamicSharedMemorySize, 64 * 1024); \
            IA_CHECK(e == hipSuccess, "route: cannot ask for shared memory: %s", hipGetErrorString(e));                 \
            asked = 1;                                                                                                  \
        }                                                                                                               \
        route_mfma_kernel<NT><<<blocks, 64 * IA_RM_WAVES, shm, stream>>>(sel, weight, (const bf16_t*)h, (const bf16_t*)router, n, W, E, top, \
                                                                         scale, score_fn, renorm, choice_bias, gates, gate_out, group_count, group_keep, plan); \
    } while (0)
        switch (nt) { case 1: IA_RM(1); break; case 2: IA_RM(2); break; case 3: IA_RM(3); break; default: IA_RM(4); break; }
#undef IA_RM
        IA_LAUNCH_CHECK("route (matrix cores)");
        return 0;
    }
    const bool vec = W % 8 == 0 && tile_mfma_aligned(h) && tile_mfma_aligned(router);
#define IA_ROUTE_SW(T, V, S, WV) route_kernel<T, V, S, WV><<<n, 64 * WV, 0, stream>>>(sel, weight, (const T*)h, (const T*)router, n, W, E, top, scale, score_fn, renorm, choice_bias, gates, gate_out, group_count, group_keep)
#define IA_ROUTE_S(T, V, S) IA_ROUTE_SW(T, V, S, IA_ROUTE_WAVES)
    // (up to 32 outputs: 8 a wave; up to 64: as many a wave as take them all in one walk over the row.  A step of few
    // tokens has few blocks, and a wave's walk is a chain of trips to the memory: sixteen waves a token then, each with
    // as few outputs as share them all out)
#define IA_ROUTE(T, V) do { if (n <= IA_ROUTE_FEW_TOKENS && E > 8) { \
            if (E <= 16) IA_ROUTE_SW(T, V, 1, 16); else if (E <= 32) IA_ROUTE_SW(T, V, 2, 16); \
            else if (E <= 48) IA_ROUTE_SW(T, V, 3, 16); else if (E <= 64) IA_ROUTE_SW(T, V, 4, 16); else IA_ROUTE_SW(T, V, 8, 16); } \
        else if (E <= 32 || E > 64) IA_ROUTE_S(T, V, 8); else if (E <= 40) IA_ROUTE_S(T, V, 10); \
        else if (E <= 48) IA_ROUTE_S(T, V, 12); else IA_ROUTE_S(T, V, 16); } while (0)
    if (dtype == IA_F32) { if (vec) IA_ROUTE(float, true); else IA_ROUTE(float, false); }
    else { if (vec) IA_ROUTE(bf16_t, true); else IA_ROUTE(bf16_t, false); }
#undef IA_ROUTE_SW
#undef IA_ROUTE_S
#undef IA_ROUTE
    IA_LAUNCH_CHECK("route");
    return 0;
}

extern "C" int ia_route_logits(int* sel, float* weight, const float* logits, long long ld, int off, int n, int E, int top, float scale,
                               int score_fn, int renorm, const float* choice_bias, int gates, float* gate_out, int group_count,
                               int group_keep, int* order, int* tile_expert, int* tile_first, int* tile_rows, int* meta, int plan_E,
                               int tile, hipStream_t stream) {
    IA_CHECK(route_groups_fit(E, top, group_count, group_keep), "route_logits: %d of %d groups of %d outputs, top %d", group_keep, group_count, E, top);
    IA_CHECK(n >= 0 && n <= IA_RM_TOKENS && E >= 1 && gates >= 0 && E + gates <= IA_MAX_EXPERTS && top >= 1 && top <= E && top <= IA_MAX_TOP &&
             off >= 0 && off + E + gates <= ld && (gates == 0 || gate_out != nullptr) && order != nullptr,
             "route_logits: n=%d (up to %d) experts=%d and %d gates at %d of rows of %lld, top=%d", n, IA_RM_TOKENS, E, gates, off, ld, top);
    IA_CHECK(score_fn == IA_SCORE_SIGMOID || score_fn == IA_SCORE_SOFTMAX, "route_logits: unknown score function %d", score_fn);
    if (n == 0) return 0;
    RoutePlan plan;
    plan.order = order; plan.tile_expert = tile_expert; plan.tile_first = tile_first; plan.tile_rows = tile_rows; plan.meta = meta;
    plan.E = plan_E; plan.tile = tile;
    route_logits_kernel<<<1, 64 * IA_RM_WAVES, 0, stream>>>(sel, weight, logits + off, ld, n, E + gates, top, scale, score_fn, renorm,
                                                            choice_bias, gates, gate_out, group_count, group_keep, plan);
    IA_LAUNCH_CHECK("route_logits");
    return 0;
}

// The most tiles of `tile` rows that `pairs` pairs over E experts can make: the grids of the two products.
static int route_tiles(int pairs, int E, int tile) { return (pairs + tile - 1) / tile + (E < pairs ? E : pairs); }
extern "C" int ia_route_tiles(int pairs, int E) { return route_tiles(pairs, E, IA_TM); }

// tile: rows of a tile, 32 (every kernel) or 64 or 128 (the matrix cores' large shapes, for many rows an expert)
extern "C" int ia_route_plan(int* order, int* tile_expert, int* tile_first, int* tile_rows, int* meta, const int* sel,
                             int pairs, int E, int tile, hipStream_t stream) {
    IA_CHECK(pairs >= 0 && E >= 1 && E <= IA_MAX_EXPERTS && (tile == 32 || tile == 64 || tile == 128), "route_plan: pairs=%d experts=%d tile=%d",
             pairs, E, tile);
    RoutePlan p;
    p.order = order; p.tile_expert = tile_expert; p.tile_first = tile_first; p.tile_rows = tile_rows; p.meta = meta; p.E = E; p.tile = tile;
    route_plan_kernel<<<1, 1024, 0, stream>>>(p, sel, pairs);
    IA_LAUNCH_CHECK("route_plan");
    return 0;
}

extern "C" int ia_experts_gate_up(void* act, const void* h, const void* w_gu, const int* order, const int* tile_expert,
                                  const int* tile_first, const int* tile_rows, const int* meta, int pairs, int E, int top,
                                  int W, int ff, float limit, float alpha, int form, int tile, int tiled, const float* in_weight,
                                  int dtype, hipStream_t stream) {
    IA_CHECK(form == IA_EXPERT_CLAMPED || form == IA_EXPERT_SILU, "experts_gate_up: unknown activation %d", form);
    IA_CHECK(pairs >= 0 && W > 0 && ff > 0 && top >= 1 && (limit > 0.f || form == IA_EXPERT_SILU) && (tile == 32 || tile == 64 || tile == 128), "experts_gate_up: bad sizes");
    if (pairs == 0) return 0;
    IA_CHECK(!tiled || (dtype == IA_BF16 && W % 8 == 0 && tile_mfma_aligned(h) && tile_mfma_aligned(w_gu)),
             "experts_gate_up: weights stored as tiles are the matrix cores' (bfloat16, widths in steps of 8)");
    IA_CHECK(tile == 32 || tiled, "experts_gate_up: tiles of 64 or 128 rows go with weights stored as tiles");
    const int features = tile == 32 ? 64 : 128;
    const dim3 grid((ff + features - 1) / features, route_tiles(pairs, E, tile));
    IA_CHECK(grid.y <= 65535, "experts_gate_up: %u row tiles are more than a grid takes", grid.y);
    if (tiled && tile == 128)
        experts_gate_up_mfma_kernel<8, 2><<<grid, 256, 0, stream>>>((bf16_t*)act, (const bf16_t*)h, (const bf16_t*)w_gu, order,
                                                                    tile_expert, tile_first, tile_rows, meta, top, W, ff, limit, alpha, form, in_weight);
    else if (tiled && tile == 64)
        experts_gate_up_mfma_kernel<4, 2><<<grid, 256, 0, stream>>>((bf16_t*)act, (const bf16_t*)h, (const bf16_t*)w_gu, order,
                                                                    tile_expert, tile_first, tile_rows, meta, top, W, ff, limit, alpha, form, in_weight);
    else if (tiled)
        experts_gate_up_mfma_kernel<2, 1><<<grid, 256, 0, stream>>>((bf16_t*)act, (const bf16_t*)h, (const bf16_t*)w_gu, order,
                                                                    tile_expert, tile_first, tile_rows, meta, top, W, ff, limit, alpha, form, in_weight);
    else if (dtype == IA_F32)
        experts_gate_up_kernel<float><<<grid, 256, 0, stream>>>((float*)act, (const float*)h, (const float*)w_gu, order,
                                                                tile_expert, tile_first, tile_rows, meta, top, W, ff, limit, alpha, form, in_weight);
    else
        experts_gate_up_kernel<bf16_t><<<grid, 256, 0, stream>>>((bf16_t*)act, (const bf16_t*)h, (const bf16_t*)w_gu, order,
                                                                 tile_expert, tile_first, tile_rows, meta, top, W, ff, limit, alpha, form, in_weight);
    IA_LAUNCH_CHECK("experts_gate_up");
    return 0;
}

extern "C" int ia_experts_down(float* y, const void* act, const void* w_down, const int* order, const int* tile_expert,
                               const int* tile_first, const int* tile_rows, const int* meta, int pairs, int E, int W,
                               int ff, int tile, int tiled, int dtype, hipStream_t stream) {
    IA_CHECK(pairs >= 0 && W > 0 && ff > 0 && (tile == 32 || tile == 64 || tile == 128), "experts_down: bad sizes");
    if (pairs == 0) return 0;
    IA_CHECK(!tiled || (dtype == IA_BF16 && ff % 8 == 0 && tile_mfma_aligned(act) && tile_mfma_aligned(w_down)),
             "experts_down: weights stored as tiles are the matrix cores' (bfloat16, widths in steps of 8)");
    IA_CHECK(tile == 32 || tiled, "experts_down: tiles of 64 or 128 rows go with weights stored as tiles");
    const int features = tile == 32 ? 64 : 128;
    const dim3 grid((W + features - 1) / features, route_tiles(pairs, E, tile));
    IA_CHECK(grid.y <= 65535, "experts_down: %u row tiles are more than a grid takes", grid.y);
    if (tiled && tile == 128)
        experts_down_mfma_kernel<8, 2><<<grid, 256, 0, stream>>>(y, (const bf16_t*)act, (const bf16_t*)w_down, order, tile_expert,
                                                                 tile_first, tile_rows, meta, W, ff);
    else if (tiled && tile == 64)
        experts_down_mfma_kernel<4, 2><<<grid, 256, 0, stream>>>(y, (const bf16_t*)act, (const bf16_t*)w_down, order, tile_expert,
                                                                 tile_first, tile_rows, meta, W, ff);
    else if (tiled)
        experts_down_mfma_kernel<2, 1><<<grid, 256, 0, stream>>>(y, (const bf16_t*)act, (const bf16_t*)w_down, order, tile_expert,
                                                                 tile_first, tile_rows, meta, W, ff);
    else if (dtype == IA_F32)
        experts_down_kernel<float><<<grid, 256, 0, stream>>>(y, (const float*)act, (const float*)w_down, order, tile_expert,
                                                             tile_first, tile_rows, meta, W, ff);
    else
        experts_down_kernel<bf16_t><<<grid, 256, 0, stream>>>(y, (const bf16_t*)act, (const bf16_t*)w_down, order, tile_expert,
                                                              tile_first, tile_rows, meta, W, ff);
    IA_LAUNCH_CHECK("experts_down");
    return 0;
}
