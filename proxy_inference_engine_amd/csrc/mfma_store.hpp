// mfma_store.hpp -- the epilogue of the one-wave-per-SIMD MFMA GEMMs (k_w16l_gemm, k_w4l2_gemm): a wave's accumulator tile, rounded, through LDS
// to whole 128-byte lines.
//
// v_mfma_f32_32x32x16 leaves register i of lane l = 32 kh + n at output column 32 nt + (i & 3) + 8 (i >> 2) + 4 kh, row 32 mi + n: a lane holds four
// consecutive columns of 32 DIFFERENT rows.  Stored from there (8 bytes per lane and row) the output cost 12-27 % of the 16-bit kernel (tower qkv
// at 4096 rows 45.5 us, 33.0 without stores; gate|up 890 vs 781): every workgroup of a round finishes at the same time and the burst is made of
// 16-byte fragments.  So the rounded tile goes through LDS -- free after the K loop; each wave its own region, rows XOR-swizzled in 8-byte slots:
// conflict-free both ways -- and leaves as 16 bytes per lane, 8 (or 4) lanes per row.
#pragma once
#include "prefill_attn.hpp"  // f32x16_t, the 16-bit traits
#include "stack_types.hpp"   // xielu

// two fp32 -> one packed pair of T in a single v_cvt_pk_* (pack2<T> converts each half separately and ORs them: 3 instructions)
template <class T>
__device__ __forceinline__ u32 w4m_pack(float lo, float hi);
template <>
__device__ __forceinline__ u32 w4m_pack<BF16>(float lo, float hi) {
    typedef float f2_t __attribute__((ext_vector_type(2)));
    typedef __bf16 b2_t __attribute__((ext_vector_type(2)));
    return __builtin_bit_cast(u32, __builtin_convertvector((f2_t){lo, hi}, b2_t));
}
template <>
__device__ __forceinline__ u32 w4m_pack<F16>(float lo, float hi) {
    typedef float f2_t __attribute__((ext_vector_type(2)));
    typedef _Float16 h2_t __attribute__((ext_vector_type(2)));
    return __builtin_bit_cast(u32, __builtin_convertvector((f2_t){lo, hi}, h2_t));
}

// acc[s][mi]: strip nt0 + s (32 columns), row block mi of the wave's tile; ot: the wave's LDS region, 32 MB x OB bytes (OB = 64 SW, or 32 SW with
// SWIGLU); m0: the tile's first row, rows: its live rows; N: the Linear's out_features (stores clipped to it), ldy: output row stride (elements);
// bias (nullable): T(T(acc) + bias), like the text tower's Linear; SWIGLU: columns (2 i, 2 i + 1) = (gate_i, up_i) -> T(T(silu(g)) * u), N / 2 wide.
// The caller has made sure nobody still reads the LDS region (a barrier after the K loop).
// ACT: MFMA_ACT_NONE, MFMA_ACT_SWIGLU (the bool true of the kernels that know only that one), MFMA_ACT_RELU2 (max(T(v), 0)^2, taken where the tile leaves LDS: next to
// the accumulators it does not fit the registers), MFMA_ACT_CLIPPED (columns paired as for SWIGLU: g sigmoid(alpha g) (u + 1) with g = min(gate, limit),
// u = clamp(up, +-limit) of the rounded pair).
// MFMA_ACT_XIELU: of the rounded value, like RELU2 on the way out of LDS (act_alpha, act_limit: its two factors).
// MFMA_ACT_GELU: columns paired as for SWIGLU: gelu_tanh(gate) up of the accumulators, with the bias, before any rounding.
enum { MFMA_ACT_NONE = 0, MFMA_ACT_SWIGLU = 1, MFMA_ACT_RELU2 = 2, MFMA_ACT_CLIPPED = 3, MFMA_ACT_XIELU = 4, MFMA_ACT_GELU = 5 };
template <class T>
__device__ __forceinline__ u32 mfma_relu2(u32 w) {
    const float a = fmaxf(lo_f32<T>(w), 0.0f), b = fmaxf(hi_f32<T>(w), 0.0f);
    return w4m_pack<T>(a * a, b * b);
}
template <class T>
__device__ __forceinline__ u32 mfma_xielu(u32 w, float up, float down) {
    return w4m_pack<T>(xielu<false>(lo_f32<T>(w), up, down), xielu<false>(hi_f32<T>(w), up, down));
}
template <class T, int MB, int SW, int ACT>
__device__ __forceinline__ void mfma_tile_store(const f32x16_t (&acc)[SW][MB], char *ot, int lane, int nt0, int m0, int rows, int N, int ldy, u16 *y,
                                                const u16 *bias, bool skip_stores = false, float act_alpha = 0.0f, float act_limit = 0.0f) {
    constexpr bool SWIGLU = ACT == MFMA_ACT_SWIGLU || ACT == MFMA_ACT_CLIPPED || ACT == MFMA_ACT_GELU;  // two columns make one
    constexpr int MT = 32 * MB;
    constexpr int OB = (SWIGLU ? 32 : 64) * SW;  // output bytes per row of the wave's tile
    constexpr int SL = OB / 8, RPB = 256 / OB;    // 8-byte slots per row; rows per 256-byte bank row
    const int n = lane & 31, kh = lane >> 5;
    const int sv = (n / RPB) & (SL - 1);  // the row's slot swizzle (rows 32 apart share it)
#pragma unroll
    for (int s = 0; s < SW; ++s) {
#pragma unroll
        for (int mi = 0; mi < MB; ++mi) {
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                const int col = 32 * (nt0 + s) + 4 * kh + 8 * q;
                if constexpr (ACT == MFMA_ACT_GELU) {  // (N is a multiple of 8: whole quads)
                    float b[4] = {0.0f, 0.0f, 0.0f, 0.0f};
                    if (bias && col < N) {
                        const uint2 w = *reinterpret_cast<const uint2 *>(bias + col);
                        b[0] = lo_f32<T>(w.x), b[1] = hi_f32<T>(w.x), b[2] = lo_f32<T>(w.y), b[3] = hi_f32<T>(w.y);
                    }
                    const float o0 = gelu_tanh<false>(acc[s][mi][4 * q] + b[0]) * (acc[s][mi][4 * q + 1] + b[1]), o1 = gelu_tanh<false>(acc[s][mi][4 * q + 2] + b[2]) * (acc[s][mi][4 * q + 3] + b[3]);
                    *reinterpret_cast<u32 *>(ot + (32 * mi + n) * OB + (((4 * s + q) ^ sv) << 3) + 4 * kh) = w4m_pack<T>(o0, o1);
                    continue;
                }
                u32 p01 = w4m_pack<T>(acc[s][mi][4 * q], acc[s][mi][4 * q + 1]), p23 = w4m_pack<T>(acc[s][mi][4 * q + 2], acc[s][mi][4 * q + 3]);  // the Linear's rounding
                if (bias && col < N) {
                    uint2 bw;
                    if (col + 4 <= N && !(N & 3)) bw = *reinterpret_cast<const uint2 *>(bias + col);
                    else {  // any out_features: the last quad of a row may be partial, rows of the bias need not be 8-byte aligned
                        u16 e[4];
#pragma unroll
                        for (int i = 0; i < 4; ++i) e[i] = col + i < N ? bias[col + i] : (u16)0;
                        bw = make_uint2(e[0] | ((u32)e[1] << 16), e[2] | ((u32)e[3] << 16));
                    }
                    p01 = w4m_pack<T>(lo_f32<T>(p01) + lo_f32<T>(bw.x), hi_f32<T>(p01) + hi_f32<T>(bw.x));
                    p23 = w4m_pack<T>(lo_f32<T>(p23) + lo_f32<T>(bw.y), hi_f32<T>(p23) + hi_f32<T>(bw.y));
                }
                char *row = ot + (32 * mi + n) * OB;
                if (SWIGLU) {  // two activations, 4 bytes at byte 32 s + 8 q + 4 kh of the row
                    const float g0 = lo_f32<T>(p01), u0 = hi_f32<T>(p01), g1 = lo_f32<T>(p23), u1 = hi_f32<T>(p23);
                    if constexpr (ACT == MFMA_ACT_CLIPPED) {
                        auto glu = [&](float g, float u) {
                            g = fminf(g, act_limit), u = fminf(fmaxf(u, -act_limit), act_limit);
                            return g / (1.0f + expf(-act_alpha * g)) * (u + 1.0f);
                        };
                        *reinterpret_cast<u32 *>(row + (((4 * s + q) ^ sv) << 3) + 4 * kh) = w4m_pack<T>(glu(g0, u0), glu(g1, u1));
                        continue;
                    }
                    const u16 o0 = T::from_f32(round_T<T>(g0 / (1.0f + expf(-g0))) * u0), o1 = T::from_f32(round_T<T>(g1 / (1.0f + expf(-g1))) * u1);
                    *reinterpret_cast<u32 *>(row + (((4 * s + q) ^ sv) << 3) + 4 * kh) = (u32)o0 | ((u32)o1 << 16);
                } else {       // 8 bytes at byte 64 s + 16 q + 8 kh
                    *reinterpret_cast<uint2 *>(row + (((8 * s + 2 * q + kh) ^ sv) << 3)) = make_uint2(p01, p23);
                }
            }
        }
    }
    // (the same wave reads what it wrote: no barrier, the compiler's lgkmcnt wait orders the LDS accesses)
    constexpr int PR = OB / 16;           // 16-byte pieces per row
    const int ldo = SWIGLU ? N >> 1 : N;  // output row length (the row stride ldy may be longer: a zero-padded operand of the next GEMM)
    const int c0 = (SWIGLU ? 16 : 32) * nt0;  // the wave's first output column
#pragma unroll
    for (int it = 0; it < MT * PR / 64; ++it) {
        const int pc = it * 64 + lane, r = pc / PR, j = pc % PR;
        const int rsv = ((r & 31) / RPB) & (SL - 1);
        uint2 lo = *reinterpret_cast<const uint2 *>(ot + r * OB + (((2 * j) ^ rsv) << 3));
        uint2 hi = *reinterpret_cast<const uint2 *>(ot + r * OB + (((2 * j + 1) ^ rsv) << 3));
        if constexpr (ACT == MFMA_ACT_RELU2) lo = make_uint2(mfma_relu2<T>(lo.x), mfma_relu2<T>(lo.y)), hi = make_uint2(mfma_relu2<T>(hi.x), mfma_relu2<T>(hi.y));
        if constexpr (ACT == MFMA_ACT_XIELU)
            lo = make_uint2(mfma_xielu<T>(lo.x, act_alpha, act_limit), mfma_xielu<T>(lo.y, act_alpha, act_limit)),
            hi = make_uint2(mfma_xielu<T>(hi.x, act_alpha, act_limit), mfma_xielu<T>(hi.y, act_alpha, act_limit));
        const int col = c0 + 8 * j;
        if (r >= rows || col >= ldo || skip_stores) continue;
        u16 *dst = y + (size_t)(m0 + r) * ldy + col;
        if (((ldo | ldy) & 7) == 0) *reinterpret_cast<uint4 *>(dst) = make_uint4(lo.x, lo.y, hi.x, hi.y);
        else if (((ldo | ldy) & 3) == 0) {  // rows are 8-byte aligned; the last piece of a row may be half
            *reinterpret_cast<uint2 *>(dst) = lo;
            if (col + 4 < ldo) *reinterpret_cast<uint2 *>(dst + 4) = hi;
        } else {  // any out_features: element by element
            const u32 w[4] = {lo.x, lo.y, hi.x, hi.y};
#pragma unroll
            for (int e = 0; e < 8; ++e)
                if (col + e < ldo) dst[e] = (u16)(w[e >> 1] >> (16 * (e & 1)));
        }
    }
}

// y = T(sum over z, in z order, of the fp32 partial tiles)
template <class T>
__global__ void __launch_bounds__(256) k_w4l_reduce(const float *part, int S, size_t MN, u16 *y) {
    const size_t i = ((size_t)blockIdx.x * 256 + threadIdx.x) * 4;
    if (i >= MN) return;
    float4 a = *reinterpret_cast<const float4 *>(part + i);
    for (int z = 1; z < S; ++z) {
        const float4 b = *reinterpret_cast<const float4 *>(part + (size_t)z * MN + i);
        a.x += b.x, a.y += b.y, a.z += b.z, a.w += b.w;
    }
    *reinterpret_cast<uint2 *>(y + i) = make_uint2(w4m_pack<T>(a.x, a.y), w4m_pack<T>(a.z, a.w));
}
