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

// One wave: the `top` experts of a row with the largest sigmoid(logit) + correction (equal ones: the first), each with the weight sigmoid(logit).
// Round k takes the best of what comes behind round k - 1's in that order, so nothing has to be marked as taken.
// put(k, expert, weight) is called by one lane, in the order of the choice.
template <class Put>
__device__ __forceinline__ void route_pick(const RouteLayer &L, const float *z, int lane, Put &&put) {
    constexpr int R = 4;  // scores a lane keeps; more experts than 64 R are scored again in every round
    float keep[R];
    auto score = [&](int e) { return 1.0f / (1.0f + expf(-z[e])) + L.correction[e]; };
#pragma unroll
    for (int r = 0; r < R; ++r) keep[r] = 64 * r + lane < L.experts ? score(64 * r + lane) : -INFINITY;
    float last = INFINITY;
    int last_e = -1;
    for (int k = 0; k < L.top; ++k) {
        float best = -INFINITY;
        int at = 0x7fffffff;
        auto look = [&](float s, int e) {
            if ((s < last || (s == last && e > last_e)) && s > best) best = s, at = e;
        };
#pragma unroll
        for (int r = 0; r < R; ++r)
            if (64 * r + lane < L.experts) look(keep[r], 64 * r + lane);
        for (int e = 64 * R + lane; e < L.experts; e += 64) look(score(e), e);
        const float top = wave_max(best);
        int e = best == top ? at : 0x7fffffff;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) e = min(e, __shfl_xor(e, o, 64));
        e = e < L.experts ? e : k;  // (scores that compare with nothing)
        last = top, last_e = e;
        if (lane == 0) put(k, e, 1.0f / (1.0f + expf(-z[e])));
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
