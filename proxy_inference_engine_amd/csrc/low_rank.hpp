// low_rank.hpp -- sixteen rows of a low-rank projection inside a workgroup of 256 threads: z[t][d] = sum_j tanh(x[t][j]) w[d][j] + b[d] for one head's channels d
// (the decays of delta_rule.hip and time_mix.hip).  bf16 stacks multiply on the matrix cores, the tanh split into bf16 halves; fp32 stacks on the vector ALU.
#pragma once
#include "stack_types.hpp"

namespace {

struct LowRankArgs {
    const void *x;      // [16][ld] T, the low-rank input's column of the first row
    int ld, rows, rank, R8;  // rows: live ones
    const u16 *bias;    // bf16 [R8], added to x; nullable
    const u16 *w;       // bf16 [D][R8]
    const float *b;     // fp32 [D]
    int D;
};

// NB: 16-channel blocks per wave.  All loads without branches around them: they leave together, and what lies outside is dropped afterwards.
template <class E, int NB>
struct LowRank {
    typedef typename E::type T;
    static constexpr bool F32 = sizeof(T) == 4;
    static constexpr int LN = 4, WS = 4;  // pairs per thread (sixteen lanes per row), weight steps: what travels ahead (ranks up to 128)
    typedef __attribute__((ext_vector_type(4))) float f32x4;
    typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
    ElemPair low[LN], lowb[LN];
    uint4 wd[F32 ? 1 : NB][WS];
    float db[NB];
    static __host__ __device__ __forceinline__ int stride(int R8) { return ((R8 + 31) & ~31) + 8; }

    static __device__ __forceinline__ ElemPair bias_at(const LowRankArgs &a, int at) {
        if (!a.bias) return {0.0f, 0.0f};
        const u32 w = *(const u32 *)(a.bias + at);
        return {lo_f32<BF16>(w), hi_f32<BF16>(w)};
    }
    static __device__ __forceinline__ ElemPair input(const LowRankArgs &a, int row, int at) { return load_pair<E>((const T *)a.x + (size_t)min(row, a.rows - 1) * a.ld + at); }
    static __device__ __forceinline__ uint4 weights(const LowRankArgs &a, int wave, int lane, int j, int s) {
        const int d = 16 * (wave * NB + j) + (lane & 15), at = 32 * s + 8 * (lane >> 4);
        const uint4 w = *(const uint4 *)(a.w + (size_t)min(d, a.D - 1) * a.R8 + min(at, a.R8 - 8));
        return d < a.D && at < a.R8 ? w : make_uint4(0, 0, 0, 0);
    }
    __device__ __forceinline__ void load(const LowRankArgs &a) {
        const int row = threadIdx.x >> 4, l = 2 * (threadIdx.x & 15);
#pragma unroll
        for (int j = 0; j < LN; ++j) {
            const int at = min(l + 32 * j, a.R8 - 2);
            low[j] = input(a, row, at), lowb[j] = bias_at(a, at);
        }
    }
    __device__ __forceinline__ void load_weights(const LowRankArgs &a, int wave, int lane) {
        if constexpr (!F32)
#pragma unroll
            for (int j = 0; j < NB; ++j) {
#pragma unroll
                for (int s = 0; s < WS; ++s) wd[j][s] = weights(a, wave, lane, j, s);
                db[j] = a.b[min(16 * (wave * NB + j) + (lane & 15), a.D - 1)];
            }
    }
    // tanh(x) into LDS: [16][stride] fp32, or two bf16 halves of that shape
    __device__ __forceinline__ void put(const LowRankArgs &a, void *lds) {
        const int row = threadIdx.x >> 4, l = 2 * (threadIdx.x & 15), LR = stride(a.R8), R32 = LR - 8;
        float *s_low = (float *)lds;
        u16 *s_hi = (u16 *)lds, *s_lo = s_hi + 16 * LR;
        auto put_pair = [&](int j, const ElemPair &v, const ElemPair &b) {
            auto f = [&](int i, float z) { return row < a.rows && i < a.rank ? stack_tanh<F32>(z) : 0.0f; };
            const float x = f(j, v.x + b.x), y = f(j + 1, v.y + b.y);
            if constexpr (F32) s_low[row * LR + j] = x, s_low[row * LR + j + 1] = y;
            else {
                const u32 hi = pack2<BF16>(x, y);
                *(u32 *)(s_hi + row * LR + j) = hi, *(u32 *)(s_lo + row * LR + j) = pack2<BF16>(x - lo_f32<BF16>(hi), y - hi_f32<BF16>(hi));
            }
        };
#pragma unroll
        for (int j = 0; j < LN; ++j)
            if (32 * j < R32) put_pair(l + 32 * j, low[j], lowb[j]);
        for (int j = l + 32 * LN; j < R32; j += 32) {
            const int at = min(j, a.R8 - 2);
            put_pair(j, input(a, row, at), bias_at(a, at));
        }
    }
    // f(t, d, z) for every row t and channel d below 16 ceil(D / 16) (channels past D: anything); behind a barrier that follows put()
    template <class F>
    __device__ __forceinline__ void product(const LowRankArgs &a, const void *lds, int wave, int lane, F &&f) {
        const int LR = stride(a.R8), R32 = LR - 8, nblk = (a.D + 15) / 16;
        if constexpr (F32) {
            const float *s_low = (const float *)lds;
            for (int i = threadIdx.x; i < 16 * 16 * nblk; i += 256) {
                const int t = i / (16 * nblk), d = i % (16 * nblk);
                float z = 0.0f;
                if (d < a.D)
                    for (int j = 0; j < a.rank; ++j) z = fmaf(s_low[t * LR + j], BF16::to_f32(a.w[(size_t)d * a.R8 + j]), z);
                f(t, d, z + a.b[min(d, a.D - 1)]);
            }
        } else {
            const u16 *s_hi = (const u16 *)lds, *s_lo = s_hi + 16 * LR;
            const int n16 = lane & 15, q = lane >> 4;
#pragma unroll
            for (int j = 0; j < NB; ++j) {
                const int b = wave * NB + j, d = 16 * b + n16;
                if (b >= nblk) break;
                f32x4 z = {0.0f, 0.0f, 0.0f, 0.0f};
                auto step = [&](int s, const uint4 &w) {
                    const uint4 hi = *(const uint4 *)(s_hi + n16 * LR + 32 * s + 8 * q), lo = *(const uint4 *)(s_lo + n16 * LR + 32 * s + 8 * q);
                    z = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, hi), __builtin_bit_cast(bf16x8, w), z, 0, 0, 0);
                    z = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, lo), __builtin_bit_cast(bf16x8, w), z, 0, 0, 0);
                };
#pragma unroll
                for (int s = 0; s < WS; ++s)
                    if (32 * s < R32) step(s, wd[j][s]);
                for (int s = WS; 32 * s < R32; ++s) step(s, weights(a, wave, lane, j, s));
#pragma unroll
                for (int i = 0; i < 4; ++i) f(4 * q + i, d, z[i] + db[j]);
            }
        }
    }
};

}  // namespace
