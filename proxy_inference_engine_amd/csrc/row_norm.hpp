// row_norm.hpp -- a row held by one workgroup, four columns per thread and pass: its loads and its norms (row_update.hip, stream_update.hip).
#pragma once
#include "stack_types.hpp"

template <int THREADS>
__device__ __forceinline__ float block_sum(float v, float *red) {  // red: THREADS / 64 floats, free again behind the next barrier
    v = lanes_sum(v);
    if constexpr (THREADS == 64) return v;
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    float s = red[0];
#pragma unroll
    for (int i = 1; i < THREADS / 64; ++i) s += red[i];
    return s;
}

__device__ __forceinline__ float4 load_quad(const void *p, bool is32, size_t row, int n, int W, int stride) {
    if (is32) {  // (fp32 rows are padded to a multiple of 64)
        return *(const float4 *)((const float *)p + row * stride + n);
    }
    const u16 *q = (const u16 *)p + row * stride + n;
    if (!(stride & 3)) {
        const uint2 v = *(const uint2 *)q;
        return make_float4(lo_f32<BF16>(v.x), hi_f32<BF16>(v.x), lo_f32<BF16>(v.y), hi_f32<BF16>(v.y));
    }
    float e[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) e[i] = n + i < W ? BF16::to_f32(q[i]) : 0.0f;
    return make_float4(e[0], e[1], e[2], e[3]);
}

// y[q] <- norm(y[q]) for the row's quads; n0 + 4 THREADS q: first column of quad q
template <int THREADS, int NQ>
__device__ __forceinline__ void norm_row(const StackNorm &m, int W, float (&y)[NQ][4], float *red) {
    const int n0 = threadIdx.x * 4;
    if (m.kind == PIE_NORM_RMS) {
        float ss = 0.0f;
#pragma unroll
        for (int q = 0; q < NQ; ++q)
#pragma unroll
            for (int i = 0; i < 4; ++i) ss = fmaf(y[q][i], y[q][i], ss);
        const float inv = 1.0f / sqrtf(block_sum<THREADS>(ss, red) / (float)W + m.param);
#pragma unroll
        for (int q = 0; q < NQ; ++q) {
            const int n = n0 + 4 * THREADS * q;
            if (n >= W) break;
            const float4 w = *(const float4 *)(m.w + n);
            y[q][0] *= inv * w.x, y[q][1] *= inv * w.y, y[q][2] *= inv * w.z, y[q][3] *= inv * w.w;
        }
    } else if (m.kind == PIE_NORM_DYN_TANH) {
        const PointNorm pn = {m.w, m.b, m.param};
#pragma unroll
        for (int q = 0; q < NQ; ++q) {
            const int n = n0 + 4 * THREADS * q;
            if (n >= W) break;
            const float4 v = point_norm4(pn, n, make_float4(y[q][0], y[q][1], y[q][2], y[q][3]));
            y[q][0] = v.x, y[q][1] = v.y, y[q][2] = v.z, y[q][3] = v.w;
        }
    }
}
