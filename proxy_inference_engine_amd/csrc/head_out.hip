// head_out.hip -- what stands between a recurrence and its output projection: every head's output (over a denominator of its own, where there is one) over its
// root mean square, times a weight and the sigmoid (or silu) of its gate.  One wave per row and HB heads; lanes own channel pairs, NP each.
#include "stack_types.hpp"

namespace {

template <class E, int NP, int HB>
__global__ void __launch_bounds__(256) k_head_out(const HeadOutArgs a, int row0) {
    typedef typename E::type T;
    constexpr bool F32 = sizeof(T) == 4;
    const size_t m = row0 + blockIdx.x;
    const int h0 = (blockIdx.y * 4 + (threadIdx.x >> 6)) * HB, lane = threadIdx.x & 63, D = a.D;
    if (h0 >= a.H) return;
    const int count = min(HB, a.H - h0);
    float2 o[HB][NP], g[HB][NP], w[HB][NP];
    float den[HB];
#pragma unroll
    for (int k = 0; k < HB; ++k) {
        den[k] = a.den ? a.den[m * a.H + h0 + min(k, count - 1)] : 1.0f;
#pragma unroll
        for (int p = 0; p < NP; ++p) {
            const int head = h0 + min(k, count - 1), d = 2 * (lane + 64 * p), dd = min(d, a.D8 - 2), at = head * a.D8 + dd;
            o[k][p] = *(const float2 *)(a.o + m * a.H * a.D8 + at);
            if (d >= D) o[k][p].x = 0.0f;
            if (d + 1 >= D) o[k][p].y = 0.0f;
            if constexpr (F32) g[k][p] = *(const float2 *)((const T *)a.gate + m * a.ldg + at);
            else {
                const u32 v = *(const u32 *)((const T *)a.gate + m * a.ldg + at);
                g[k][p] = make_float2(lo_f32<BF16>(v), hi_f32<BF16>(v));
            }
            if (a.gate_bias) {
                const u32 v = *(const u32 *)(a.gate_bias + at);
                g[k][p].x += lo_f32<BF16>(v), g[k][p].y += hi_f32<BF16>(v);
            }
            const float *wh = a.w + (a.shared_w ? 0 : head * D);
            w[k][p] = make_float2(wh[min(d, D - 1)], wh[min(d + 1, D - 1)]);
        }
    }
    const float inv_d = 1.0f / (float)D;
#pragma unroll
    for (int k = 0; k < HB; ++k) {
        if (k >= count) break;
        if (a.den) {
            const float r = 1.0f / den[k];
#pragma unroll
            for (int p = 0; p < NP; ++p) o[k][p].x *= r, o[k][p].y *= r;
        }
        float ss = 0.0f;
#pragma unroll
        for (int p = 0; p < NP; ++p) ss = fmaf(o[k][p].x, o[k][p].x, fmaf(o[k][p].y, o[k][p].y, ss));
        ss = lanes_sum(ss) * inv_d + a.eps;
        const float inv = F32 ? 1.0f / sqrtf(ss) : __builtin_amdgcn_rsqf(ss);
        T *out = (T *)a.out + m * a.ld_out + (h0 + k) * a.D8;
#pragma unroll
        for (int p = 0; p < NP; ++p) {
            const int d = 2 * (lane + 64 * p);
            if (d >= D) break;
            float x = o[k][p].x * inv * w[k][p].x * stack_sigmoid<F32>(g[k][p].x), y = o[k][p].y * inv * w[k][p].y * stack_sigmoid<F32>(g[k][p].y);  // (past an odd head's end: zero)
            x *= a.silu ? g[k][p].x * a.scale : a.scale, y *= a.silu ? g[k][p].y * a.scale : a.scale;
            if constexpr (F32) *(float2 *)(out + d) = make_float2(x, y);
            else *(u32 *)(out + d) = pack2<BF16>(x, y);
        }
    }
}

template <class E>
void head_out_go(const HeadOutArgs &a, int row0, int rows, hipStream_t st) {
    const bool few = rows < 64;  // (few rows: a wave per head)
#define HO_GO(NP_, HB_) hipLaunchKernelGGL((k_head_out<E, NP_, HB_>), dim3((unsigned)rows, (unsigned)((a.H + 4 * HB_ - 1) / (4 * HB_))), dim3(256), 0, st, a, row0)
    if (a.D <= 128) {
        if (few) HO_GO(1, 1);
        else HO_GO(1, 8);
    } else if (a.D <= 256) {
        if (few) HO_GO(2, 1);
        else HO_GO(2, 4);
    } else if (a.D <= 512) {
        if (few) HO_GO(4, 1);
        else HO_GO(4, 2);
    } else HO_GO(16, 1);
#undef HO_GO
}

}  // namespace

int head_out_launch(int dtype, const HeadOutArgs &a, int row0, int rows, hipStream_t st) {
    if (rows <= 0) return PIE_OK;
    PIE_REQUIRE(a.D > 0 && a.D <= HEAD_OUT_MAX_DIM && a.H > 0, PIE_E_SHAPE, "head outputs: heads of at most 2048 numbers");
    if (dtype == PIE_F32) head_out_go<ElemF32>(a, row0, rows, st);
    else head_out_go<ElemBF16>(a, row0, rows, st);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}
