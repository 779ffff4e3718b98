// route.hpp -- which rows a mixture's experts get: a router's choice, and the row lists by expert.
#pragma once
#include "stack_types.hpp"

struct RouteLayer {      // one mixture layer's row lists (device pointers)
    const int *table;    // experts by token id; nullptr: by the router's logits
    const float *logits, *correction;  // [M][ld_logits], [experts]
    int ld_logits;
    int *chosen;         // [M * top]: the router's choice, best first, and the weights
    float *weight;
    int top, experts, max_active;
    int *active, *offset, *list, *place;  // [max_active], [experts + 1], [M * top] rows by expert, [M * top] position of (row, slot)
    int4 *tiles;  // {expert, first position, rows, 0}: row tiles of the grouped GEMM
};

constexpr int ROUTE_KEPT = 4;  // scores a lane keeps: up to 64 ROUTE_KEPT experts
__device__ __forceinline__ void route_corrections(const RouteLayer &L, int lane, float (&corr)[ROUTE_KEPT]) {
#pragma unroll
    for (int r = 0; r < ROUTE_KEPT; ++r) corr[r] = L.correction[min(64 * r + lane, L.experts - 1)];
}
// One wave: the `top` experts of a row with the largest sigmoid(logit) + correction (equal ones: the first), each with the weight sigmoid(logit).
// corr: what route_corrections() read.  put(k, expert, weight) is called by all lanes with the same arguments, in the order of the choice.
template <class Put>
__device__ __forceinline__ void route_pick(const RouteLayer &L, const float *z, int lane, const float (&corr)[ROUTE_KEPT], Put &&put) {
    constexpr int R = ROUTE_KEPT;
    auto sigmoid = [&](int e) { return 1.0f / (1.0f + expf(-z[e])); };
    if (L.experts <= 64 * R) {  // a chosen score is taken out
        float keep[R];
#pragma unroll
        for (int r = 0; r < R; ++r) keep[r] = 64 * r + lane < L.experts ? sigmoid(64 * r + lane) + corr[r] : -INFINITY;
        for (int k = 0; k < L.top; ++k) {
            const float top = lanes_max(fmaxf(fmaxf(keep[0], keep[1]), fmaxf(keep[2], keep[3])));
            int e = L.experts;
#pragma unroll
            for (int r = R - 1; r >= 0; --r) {
                const unsigned long long has = __ballot(keep[r] == top);
                if (has) e = 64 * r + __builtin_ctzll(has);
            }
            e = e < L.experts ? e : k;  // (scores that compare with nothing)
#pragma unroll
            for (int r = 0; r < R; ++r)
                if (64 * r + lane == e) keep[r] = -INFINITY;
            put(k, e, sigmoid(e));
        }
        return;
    }
    // many experts: scored again in every round, which takes the best of what comes behind the round before in the order of the choice
    float last = INFINITY;
    int last_e = -1;
    for (int k = 0; k < L.top; ++k) {
        float best = -INFINITY;
        int at = 0x7fffffff;
        for (int e = lane; e < L.experts; e += 64) {
            const float s = sigmoid(e) + L.correction[e];
            if ((s < last || (s == last && e > last_e)) && s > best) best = s, at = e;
        }
        const float top = lanes_max(best);
        int e = best == top ? at : 0x7fffffff;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) e = min(e, __shfl_xor(e, o, 64));
        e = e < L.experts ? e : k;
        last = top, last_e = e;
        put(k, e, sigmoid(e));
    }
}

// One wave: the lists of a single row, without counting: every chosen expert has it, in the order of their numbers.  top <= 64.
__device__ __forceinline__ void route_single(const RouteLayer &L, const float *z, int lane, const float (&corr)[ROUTE_KEPT]) {
    int mine = 0x7fffffff, rank = 0;
    float weight = 0.0f;
    route_pick(L, z, lane, corr, [&](int k, int e, float w) {
        if (lane == k) mine = e, weight = w;
    });
    for (int k = 0; k < L.top; ++k) rank += __builtin_amdgcn_readlane(mine, k) < mine;
    if (lane < L.top) {
        L.weight[lane] = weight, L.place[lane] = rank, L.list[rank] = 0, L.active[rank] = mine;
        L.offset[mine] = rank, L.offset[mine + 1] = rank + 1;  // (neighbours that are both chosen agree)
    }
}

// The row lists of one mixture, by a whole workgroup: expert(i) names the expert of (row, slot) i.  s_cnt: 2 * experts ints of LDS.
// With L.tiles, also the row tiles of the grouped GEMM: tr rows each, in blocks of rb, max_tiles entries.
template <class F>
__device__ __forceinline__ void route_lists(const RouteLayer &L, int M, int *s_cnt, F &&named, int tr, int rb, int max_tiles) {
    int *s_cur = s_cnt + L.experts;
    const int n = M * L.top;
    auto expert = [&](int i) { return min(max(named(i), 0), L.experts - 1); };
    for (int e = threadIdx.x; e < L.experts; e += blockDim.x) s_cnt[e] = 0;
    __syncthreads();
    for (int i = threadIdx.x; i < n; i += blockDim.x) atomicAdd(&s_cnt[expert(i)], 1);
    __syncthreads();
    if (threadIdx.x < 64) {
        int base = 0, n_active = 0, n_tiles = 0;
        for (int e0 = 0; e0 < L.experts; e0 += 64) {
            const int e = e0 + (int)threadIdx.x, c = e < L.experts ? s_cnt[e] : 0;
            int incl = c;
#pragma unroll
            for (int o = 1; o < 64; o <<= 1) {
                const int v = __shfl_up(incl, o, 64);
                if ((int)threadIdx.x >= o) incl += v;
            }
            if (e < L.experts) s_cur[e] = L.offset[e] = base + incl - c;
            const unsigned long long has = __ballot(c > 0);
            const int slot = n_active + __popcll(has & ((1ull << threadIdx.x) - 1ull));
            if (c > 0 && slot < L.max_active) L.active[slot] = e;
            if (max_tiles) {
                const int mine = (c + tr - 1) / tr, slots = (mine + rb - 1) / rb * rb;
                int ti = slots;
#pragma unroll
                for (int o = 1; o < 64; o <<= 1) {
                    const int v = __shfl_up(ti, o, 64);
                    if ((int)threadIdx.x >= o) ti += v;
                }
                for (int k = 0; k < slots; ++k) L.tiles[n_tiles + ti - slots + k] = make_int4(e, base + incl - c + k * tr, max(0, min(tr, c - k * tr)), 0);
                n_tiles += __shfl(ti, 63, 64);
            }
            base += __shfl(incl, 63, 64), n_active += __popcll(has);
        }
        for (int i = n_tiles + (int)threadIdx.x; i < max_tiles; i += 64) L.tiles[i] = make_int4(0, 0, 0, 0);
        if (threadIdx.x == 0) L.offset[L.experts] = base;
        for (int i = n_active + (int)threadIdx.x; i < L.max_active; i += 64) L.active[i] = -1;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < n; i += blockDim.x) {
        const int p = atomicAdd(&s_cur[expert(i)], 1);
        L.list[p] = i / L.top;
        L.place[i] = p;
    }
}
