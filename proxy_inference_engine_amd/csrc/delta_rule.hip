// delta_rule.hip -- the generalised delta rule (PIE_MIXER_DELTA): per head a state S [key channel][value column] in fp32, carried from token to token,
//   S_t = diag(w_t) S_(t-1) - (a_t u_t) (u_t^T S_(t-1)) + k_t v_t^T,   o_t = S_t^T r_t,
// with the unit key u = k / sqrt(sum k^2 + unit_eps), the decay w = exp(-decay_scale sigmoid(.)) and the removal rate a = sigmoid(.), all fp32.
//
// Step form (decoded tokens, short runs): one workgroup per (run, head).  A thread keeps RPT key channels of one value column in registers; the channel
// vectors of a token are broadcast from LDS.  Columns are independent, so a token costs two exchanges between the channel slices: u^T S and r^T S.
// The decay's low-rank projection, the unit key, the head's norm and the output gate are taken on the way.
//
// Chunk form (longer runs), 16 tokens at a time on the fp32 matrix cores.  With W_t the product of the decays up to t inside a chunk, S the state in front of
// it and p_t = S_(t-1)^T u_t what token t removes,
//   p_t = S^T (W_(t-1) u_t) + sum_{i<t} A_ti v_i - sum_{i<t} B_ti p_i,     A_ti = u_t^T (W_(t-1) / W_i) k_i,   B_ti = u_t^T (W_(t-1) / W_i) a_i u_i
//   o_t = S^T (W_t r_t) + sum_{i<=t} A'_ti v_i - sum_{i<=t} B'_ti p_i,     A', B' likewise with r_t and W_t
//   S  <- W_16 S + sum_i (W_16 / W_i) (k_i v_i^T - a_i u_i p_i^T)
// Everything but S and p is known beforehand: one launch (all chunks of all heads in parallel) takes the channel vectors, A, B, A', B' and T = (I + B)^-1 and
// leaves T U, R, K, -A and T A, A', -B' in matrix operand order; a second walks the chunks, one workgroup per head and 16 value columns, whose four waves
// split the key channels of S (which stays in accumulators and is its own B operand); a third takes the heads' norm and gate.  Decays are above exp(-0.61), so
// W_16 > 6e-5: the quotients are formed as W_t times 1 / W_i in fp32 without loss.
#include <algorithm>

#include "stack_types.hpp"

typedef __attribute__((ext_vector_type(4))) float dr_f32x4;
typedef __attribute__((ext_vector_type(8))) __bf16 dr_bf16x8;

namespace {

constexpr int DC = 16;  // tokens of a chunk


template <class E, int CP, int NT>  // CP: power of two >= D; NT threads
__global__ void __launch_bounds__(NT) k_delta_step(const DeltaArgs a) {
    typedef typename E::type T;
    constexpr int SL = NT / CP, RPT = CP / SL;  // channel slices; channels per thread
    static_assert(NT % CP == 0 && CP % SL == 0 && NT % 64 == 0, "slices");
    __shared__ __attribute__((aligned(16))) float s_r[CP], s_k[CP], s_v[CP], s_g[CP], s_a[CP], s_w[CP], s_low[DELTA_MAX_RANK], s_p[SL][CP], s_o[SL][CP], s_ss[NT / 64];
    const int run_i = blockIdx.x, head = blockIdx.y, D = a.D, lane = threadIdx.x & 63;
    const RowRun run = a.runs[run_i];
    const int col = threadIdx.x % CP, slice = threadIdx.x / CP, d0 = slice * RPT;
    const int seq = min(a.row_seq[run.row0], a.n_seqs - 1);
    const size_t slot = min((unsigned)a.slots[seq], (unsigned)a.n_slots - 1u);
    float *state = a.state + (slot * a.H + head) * D * D;
    float S[RPT];
    const bool fresh = a.pos[run.row0] == 0;
#pragma unroll
    for (int i = 0; i < RPT; ++i) S[i] = !fresh && col < D && d0 + i < D ? state[(size_t)(d0 + i) * D + col] : 0.0f;
    const int HD8 = a.H * a.D8;

    for (int j = 0; j < run.n_rows; ++j) {
        const size_t m = run.row0 + j;
        const T *x = (const T *)a.raw + m * a.ld + head * a.D8;
        const u16 *bias = a.bias ? a.bias + head * a.D8 : nullptr;
        for (int i = threadIdx.x; i < 5 * CP; i += NT) {  // r, k, v, gate, rate; channels past D: nothing
            const int what = i / CP, d = i % CP;
            float v = d < D ? E::load(x + what * HD8 + d) + (bias ? BF16::to_f32(bias[what * HD8 + d]) : 0.0f) : 0.0f;
            if (what >= 3) v = d < D ? 1.0f / (1.0f + expf(-v)) : 0.0f;
            float *dst = what == 0 ? s_r : what == 1 ? s_k : what == 2 ? s_v : what == 3 ? s_g : s_a;
            dst[d] = v;
        }
        for (int i = threadIdx.x; i < a.R8; i += NT) {
            const float z = i < a.rank ? E::load((const T *)a.raw + m * a.ld + 5 * HD8 + i) + (a.bias ? BF16::to_f32(a.bias[5 * HD8 + i]) : 0.0f) : 0.0f;
            s_low[i] = tanhf(z);
        }
        __syncthreads();
        // the decay: eight lanes per channel
        for (int d = threadIdx.x >> 3; d < CP; d += NT / 8) {
            float z = 0.0f;
            if (d < D) {
                const u16 *wr = a.w_decay + (size_t)(head * D + d) * a.R8;
                for (int i = (threadIdx.x & 7) * 8; i < a.R8; i += 64) {
                    const uint4 q = *(const uint4 *)(wr + i);
                    const float4 l0 = *(const float4 *)(s_low + i), l1 = *(const float4 *)(s_low + i + 4);
                    z = fmaf(lo_f32<BF16>(q.x), l0.x, fmaf(hi_f32<BF16>(q.x), l0.y, fmaf(lo_f32<BF16>(q.y), l0.z, fmaf(hi_f32<BF16>(q.y), l0.w, z))));
                    z = fmaf(lo_f32<BF16>(q.z), l1.x, fmaf(hi_f32<BF16>(q.z), l1.y, fmaf(lo_f32<BF16>(q.w), l1.z, fmaf(hi_f32<BF16>(q.w), l1.w, z))));
                }
            }
            z = lanes8_sum(z);
            if ((threadIdx.x & 7) == 0) s_w[d] = d < D ? expf(-a.decay_scale / (1.0f + expf(-(z + a.decay_bias[head * D + d])))) : 1.0f;
        }
        float ss = 0.0f;  // every wave: the key's length
        for (int d = lane; d < CP; d += 64) ss = fmaf(s_k[d], s_k[d], ss);
        const float unit = 1.0f / sqrtf(wave_sum(ss) + a.unit_eps);
        float p = 0.0f;
#pragma unroll
        for (int i = 0; i < RPT; ++i) p = fmaf(s_k[d0 + i], S[i], p);
        s_p[slice][col] = p * unit;
        __syncthreads();
        p = 0.0f;
#pragma unroll
        for (int i = 0; i < SL; ++i) p += s_p[i][col];
        const float v = s_v[col];
        float o = 0.0f;
#pragma unroll
        for (int i = 0; i < RPT; ++i) {
            const float k = s_k[d0 + i];
            S[i] = fmaf(k, v, fmaf(-(s_a[d0 + i] * k * unit), p, s_w[d0 + i] * S[i]));
            o = fmaf(s_r[d0 + i], S[i], o);
        }
        s_o[slice][col] = o;
        __syncthreads();
        if (threadIdx.x < (CP < 64 ? 64 : CP)) {  // whole waves
            o = 0.0f;
            if (threadIdx.x < CP)
#pragma unroll
                for (int i = 0; i < SL; ++i) o += s_o[i][col];
            const float sum = wave_sum(o * o);
            if (lane == 0) s_ss[threadIdx.x >> 6] = sum;
        }
        __syncthreads();
        if (threadIdx.x < D) {
            float sum = s_ss[0];
#pragma unroll
            for (int i = 1; i < (CP + 63) / 64; ++i) sum += s_ss[i];
            const float y = o * (1.0f / sqrtf(sum / (float)D + a.eps)) * a.o_norm[head * D + threadIdx.x] * s_g[threadIdx.x];
            ((T *)a.out)[m * a.ld_out + head * a.D8 + threadIdx.x] = E::pack(y);
        }
        __syncthreads();  // the channel vectors are written again
    }
    if (col < D)
#pragma unroll
        for (int i = 0; i < RPT; ++i)
            if (d0 + i < D) state[(size_t)(d0 + i) * D + col] = S[i];
}

// ---------------------------------------------------------------- chunk form
__host__ __device__ __forceinline__ int dr_blocks(int D) { return (D + 15) / 16; }
// per (chunk, head): T U, R, K, -A [blocks][64 lanes][4] each; T A, A', -B' [64][4]; W_16 [16 blocks]
__host__ __device__ __forceinline__ size_t dr_chunk_floats(int D) { return (size_t)dr_blocks(D) * (4 * 256 + 16) + 3 * 256; }

__device__ __forceinline__ dr_f32x4 dr_mfma(float a, float b, const dr_f32x4 &c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

struct DeltaChunk {
    int row0, n;  // rows [row0, row0 + n)
};
__device__ __forceinline__ DeltaChunk dr_chunk(const DeltaArgs &a, int i) {
    int r = 0;
    for (;;) {
        const int n = (a.runs[r].n_rows + DC - 1) / DC;
        if (i < n || r + 1 >= a.n_runs) break;
        i -= n, ++r;
    }
    return {a.runs[r].row0 + DC * i, min(DC, a.runs[r].n_rows - DC * i)};
}

// NB: 16-channel blocks per wave (D <= 64 NB).  Dynamic LDS: see delta_prep_lds().
template <class E, int NB>
__global__ void __launch_bounds__(256) k_delta_prep(const DeltaArgs a) {
    typedef typename E::type T;
    constexpr bool F32 = sizeof(T) == 4;
    constexpr int LD = 64 * NB + 4, CH = 64 * NB, PARTS = 256 / CH, TP = DC / PARTS, LM = 20;
    extern __shared__ __attribute__((aligned(16))) char lds[];
    float *s_l = (float *)lds, *s_m = s_l + DC * LD, *s_unit = s_m + 5 * DC * LM, *s_wc = s_unit + DC;  // log decays; A, B, A', B', T; 1 / |k|; W_16
    float *s_u = s_wc + CH, *s_r = s_u + DC * LD, *s_k = s_r + DC * LD, *s_a = s_k + DC * LD;
    // (the low-rank input of the decay lies where the channel vectors come later)
    const int D = a.D, nblk = dr_blocks(D), lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), n16 = lane & 15, q = lane >> 4;
    const int head = blockIdx.y, HD8 = a.H * a.D8;
    const DeltaChunk c = dr_chunk(a, blockIdx.x);
    if (c.n <= 0) return;
    const T *raw = (const T *)a.raw + (size_t)c.row0 * a.ld;
    const int R32 = (a.R8 + 31) & ~31, LR = R32 + 8;
    u16 *s_hi = (u16 *)s_u, *s_lo = s_hi + DC * LR;
    float *s_low = s_u;
    for (int i = threadIdx.x; i < DC * R32; i += 256) {
        const int t = i / R32, j = i % R32;
        const float v = t < c.n && j < a.rank ? tanhf(E::load(raw + (size_t)t * a.ld + 5 * HD8 + j) + (a.bias ? BF16::to_f32(a.bias[5 * HD8 + j]) : 0.0f)) : 0.0f;
        if constexpr (F32) s_low[t * LR + j] = v;
        else {
            const u16 hi = BF16::from_f32(v);
            s_hi[t * LR + j] = hi, s_lo[t * LR + j] = BF16::from_f32(v - BF16::to_f32(hi));
        }
    }
    const T *x = raw + head * a.D8;  // this head's r; k, v, gate, rate behind it at HD8 each
    const u16 *bias = a.bias ? a.bias + head * a.D8 : nullptr;
    auto channel = [&](int what, int t, int d) { return E::load(x + (size_t)t * a.ld + what * HD8 + d) + (bias ? BF16::to_f32(bias[what * HD8 + d]) : 0.0f); };
    {
        const int t = threadIdx.x >> 4;
        float ss = 0.0f;
        if (t < c.n)
            for (int d = threadIdx.x & 15; d < D; d += 16) {
                const float k = channel(1, t, d);
                ss = fmaf(k, k, ss);
            }
        ss = lanes16_sum(ss);
        if ((threadIdx.x & 15) == 0) s_unit[t] = 1.0f / sqrtf(ss + a.unit_eps);
    }
    __syncthreads();
    auto log_decay = [&](int t, int d, float z) { s_l[t * LD + d] = t < c.n && d < D ? -a.decay_scale / (1.0f + expf(-(z + a.decay_bias[head * D + min(d, D - 1)]))) : 0.0f; };
    if constexpr (F32) {
        for (int i = threadIdx.x; i < DC * 16 * nblk; i += 256) {
            const int t = i / (16 * nblk), d = i % (16 * nblk);
            float z = 0.0f;
            if (d < D)
                for (int j = 0; j < a.rank; ++j) z = fmaf(s_low[t * LR + j], BF16::to_f32(a.w_decay[(size_t)(head * D + d) * a.R8 + j]), z);
            log_decay(t, d, z);
        }
    } else {
#pragma unroll
        for (int j = 0; j < NB; ++j) {
            const int b = wave * NB + j, d = 16 * b + n16;
            if (b >= nblk) break;
            dr_f32x4 z = {0.0f, 0.0f, 0.0f, 0.0f};
            for (int s = 0; s < R32; s += 32) {
                const int at = s + 8 * q;
                const uint4 w = d < D && at < a.R8 ? *(const uint4 *)(a.w_decay + (size_t)(head * D + d) * a.R8 + at) : make_uint4(0, 0, 0, 0);
                const uint4 hi = *(const uint4 *)(s_hi + n16 * LR + at), lo = *(const uint4 *)(s_lo + n16 * LR + at);
                z = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(dr_bf16x8, hi), __builtin_bit_cast(dr_bf16x8, w), z, 0, 0, 0);
                z = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(dr_bf16x8, lo), __builtin_bit_cast(dr_bf16x8, w), z, 0, 0, 0);
            }
#pragma unroll
            for (int i = 0; i < 4; ++i) log_decay(4 * q + i, d, z[i]);
        }
    }
    __syncthreads();  // the low-rank input has been read
    {
        const int d = threadIdx.x % CH, part = threadIdx.x / CH;
        if (part < PARTS && d < 16 * nblk) {
            float L = 0.0f;
            for (int t = 0; t < part * TP; ++t) L += s_l[t * LD + d];
#pragma unroll
            for (int j = 0; j < TP; ++j) {
                const int t = part * TP + j;
                const bool live = t < c.n && d < D;
                const float before = expf(L);
                L += s_l[t * LD + d];
                const float e = expf(L), back = expf(-L);
                float r = 0.0f, k = 0.0f, ra = 0.0f;
                if (live) r = channel(0, t, d), k = channel(1, t, d), ra = 1.0f / (1.0f + expf(-channel(4, t, d)));
                const float u = k * s_unit[t];
                s_u[t * LD + d] = u * before, s_r[t * LD + d] = r * e, s_k[t * LD + d] = k * back, s_a[t * LD + d] = ra * u * back;
            }
            if (part == PARTS - 1) s_wc[d] = expf(L);
        }
    }
    __syncthreads();
    {  // wave 0: A = U K^T, 1: B = U A^T, 2: A' = R K^T, 3: B' = R A^T
        const float *l = wave < 2 ? s_u : s_r, *r = wave & 1 ? s_a : s_k;
        dr_f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
        for (int b = 0; b < nblk; ++b) {
            const dr_f32x4 lv = *(const dr_f32x4 *)(l + n16 * LD + 16 * b + 4 * q), rv = *(const dr_f32x4 *)(r + n16 * LD + 16 * b + 4 * q);
#pragma unroll
            for (int i = 0; i < 4; ++i) acc = dr_mfma(lv[i], rv[i], acc);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) s_m[(wave * DC + 4 * q + i) * LM + n16] = n16 < 4 * q + i + (wave >= 2) ? acc[i] : 0.0f;
    }
    __syncthreads();
    float *out = a.ws + ((size_t)blockIdx.x * a.H + head) * dr_chunk_floats(D);
    float *o_r = out + nblk * 256, *o_k = o_r + nblk * 256, *o_a = o_k + nblk * 256, *o_m = o_a + nblk * 256;
    float *s_t = s_m + 4 * DC * LM;
    if (wave == 0) {
        float tc[DC];  // column n16 of (I + B)^-1
#pragma unroll
        for (int t = 0; t < DC; ++t) {
            float v = t == n16 ? 1.0f : 0.0f;
#pragma unroll
            for (int i = 0; i < t; ++i) v = fmaf(-s_m[(DC + t) * LM + i], tc[i], v);
            tc[t] = v;
        }
        if (q == 0)
#pragma unroll
            for (int t = 0; t < DC; ++t) s_t[t * LM + n16] = tc[t];
        dr_f32x4 ta = {0.0f, 0.0f, 0.0f, 0.0f};
        const dr_f32x4 tv = *(const dr_f32x4 *)(s_t + n16 * LM + 4 * q);
#pragma unroll
        for (int i = 0; i < 4; ++i) ta = dr_mfma(s_m[(4 * q + i) * LM + n16], tv[i], ta);  // (T A)^T
        *(dr_f32x4 *)(o_m + lane * 4) = ta;
    } else {
        for (int b = wave - 1; b < nblk; b += 3) {
            *(dr_f32x4 *)(o_r + b * 256 + lane * 4) = *(const dr_f32x4 *)(s_r + n16 * LD + 16 * b + 4 * q);
            const float w = s_wc[16 * b + n16];
            dr_f32x4 k, m;
#pragma unroll
            for (int i = 0; i < 4; ++i) k[i] = s_k[(4 * q + i) * LD + 16 * b + n16] * w, m[i] = -s_a[(4 * q + i) * LD + 16 * b + n16] * w;
            *(dr_f32x4 *)(o_k + b * 256 + lane * 4) = k, *(dr_f32x4 *)(o_a + b * 256 + lane * 4) = m;
        }
        if (wave == 2) *(dr_f32x4 *)(o_m + 256 + lane * 4) = *(const dr_f32x4 *)(s_m + (2 * DC + n16) * LM + 4 * q);
        if (wave == 3) *(dr_f32x4 *)(o_m + 512 + lane * 4) = -*(const dr_f32x4 *)(s_m + (3 * DC + n16) * LM + 4 * q);
        if (wave == 1)
            for (int d = lane; d < 16 * nblk; d += 64) o_m[768 + d] = s_wc[d];
    }
    __syncthreads();
    const dr_f32x4 tv = *(const dr_f32x4 *)(s_t + n16 * LM + 4 * q);
#pragma unroll
    for (int j = 0; j < NB; ++j) {
        const int b = wave * NB + j;
        if (b >= nblk) break;
        dr_f32x4 u = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int i = 0; i < 4; ++i) u = dr_mfma(s_u[(4 * q + i) * LD + 16 * b + n16], tv[i], u);  // (T U)^T
        *(dr_f32x4 *)(out + b * 256 + lane * 4) = u;
    }
}

template <class E, int NB>
__global__ void __launch_bounds__(256) k_delta_scan(const DeltaArgs a) {
    typedef typename E::type T;
    __shared__ dr_f32x4 s_p[2][4][64], s_o[2][4][64];
    const int D = a.D, nblk = dr_blocks(D), lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), n16 = lane & 15, q = lane >> 4;
    const int head = (int)blockIdx.x % a.H, cb = (int)blockIdx.x / a.H, col = 16 * cb + n16;  // (head fastest: the column blocks of a head share an L2 where H is a multiple of 8)
    const RowRun run = a.runs[blockIdx.y];
    int chunk0 = 0;
    for (int r = 0; r < (int)blockIdx.y; ++r) chunk0 += (a.runs[r].n_rows + DC - 1) / DC;
    const int chunks = (run.n_rows + DC - 1) / DC;
    const size_t slot = min((unsigned)a.slots[min(a.row_seq[run.row0], a.n_seqs - 1)], (unsigned)a.n_slots - 1u);
    float *state = a.state + (slot * a.H + head) * D * D;
    const bool fresh = a.pos[run.row0] == 0;
    dr_f32x4 S[NB];  // S[16 b + 4 q + i][col]
#pragma unroll
    for (int j = 0; j < NB; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int d = 16 * (wave * NB + j) + 4 * q + i;
            S[j][i] = !fresh && d < D && col < D ? state[(size_t)d * D + col] : 0.0f;
        }
    const size_t per = dr_chunk_floats(D);
    const float *ws = a.ws + ((size_t)chunk0 * a.H + head) * per;
    const T *vp = (const T *)a.raw + (size_t)run.row0 * a.ld + 2 * a.H * a.D8 + head * a.D8 + min(col, D - 1);
    const float vbias = a.bias ? BF16::to_f32(a.bias[2 * a.H * a.D8 + head * a.D8 + min(col, D - 1)]) : 0.0f;
    struct Operands {
        dr_f32x4 u[NB], r[NB], k[NB], m[NB], w[NB], v, x;  // x: T A (wave 0), A' (wave 1), -B' (wave 2)
    };
    const dr_f32x4 zero = {0.0f, 0.0f, 0.0f, 0.0f};
    auto load = [&](int c, Operands &o) {
        const float *p = ws + (size_t)c * a.H * per;
#pragma unroll
        for (int j = 0; j < NB; ++j) {
            const int b = wave * NB + j;
            if (b < nblk) {
                const float *pb = p + b * 256 + lane * 4;
                o.u[j] = *(const dr_f32x4 *)pb, o.r[j] = *(const dr_f32x4 *)(pb + nblk * 256), o.k[j] = *(const dr_f32x4 *)(pb + 2 * nblk * 256), o.m[j] = *(const dr_f32x4 *)(pb + 3 * nblk * 256);
                o.w[j] = *(const dr_f32x4 *)(p + nblk * 1024 + 768 + 16 * b + 4 * q);
            } else o.u[j] = o.r[j] = o.k[j] = o.m[j] = o.w[j] = zero;
        }
        o.x = *(const dr_f32x4 *)(p + nblk * 1024 + min(wave, 2) * 256 + lane * 4);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = DC * c + 4 * q + i;
            const float v = E::load(vp + (size_t)min(t, run.n_rows - 1) * a.ld) + vbias;
            o.v[i] = t < run.n_rows && col < D ? v : 0.0f;
        }
    };
    auto store_o = [&](int c) {  // chunk c's outputs: one per thread
        const float *p = (const float *)s_o[c & 1] + threadIdx.x;
        const float o = (p[0] + p[256]) + (p[512] + p[768]);
        const int l = threadIdx.x >> 2, t = DC * c + 4 * (l >> 4) + (threadIdx.x & 3), d = 16 * cb + (l & 15);
        if (t < run.n_rows && d < D) a.o[((size_t)(run.row0 + t) * a.H + head) * a.D8 + d] = o;
    };
    auto step = [&](int c, const Operands &o) {
        dr_f32x4 P = zero, O = zero;
#pragma unroll
        for (int j = 0; j < NB; ++j)
#pragma unroll
            for (int i = 0; i < 4; ++i) P = dr_mfma(o.u[j][i], S[j][i], P);
        if (wave == 0)
#pragma unroll
            for (int i = 0; i < 4; ++i) P = dr_mfma(o.x[i], o.v[i], P);
        s_p[c & 1][wave][lane] = P;
#pragma unroll
        for (int j = 0; j < NB; ++j)
#pragma unroll
            for (int i = 0; i < 4; ++i) O = dr_mfma(o.r[j][i], S[j][i], O);
        if (wave == 1)
#pragma unroll
            for (int i = 0; i < 4; ++i) O = dr_mfma(o.x[i], o.v[i], O);
#pragma unroll
        for (int j = 0; j < NB; ++j) S[j] *= o.w[j];
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int j = 0; j < NB; ++j) S[j] = dr_mfma(o.k[j][i], o.v[i], S[j]);
        __syncthreads();
        P = (s_p[c & 1][0][lane] + s_p[c & 1][1][lane]) + (s_p[c & 1][2][lane] + s_p[c & 1][3][lane]);
        if (c > 0) store_o(c - 1);
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int j = 0; j < NB; ++j) S[j] = dr_mfma(o.m[j][i], P[i], S[j]);
        if (wave == 2)
#pragma unroll
            for (int i = 0; i < 4; ++i) O = dr_mfma(o.x[i], P[i], O);
        s_o[c & 1][wave][lane] = O;
    };
    Operands even, odd;
    load(0, even);
    for (int c = 0; c < chunks; c += 2) {
        load(min(c + 1, chunks - 1), odd);
        step(c, even);
        if (c + 1 >= chunks) break;
        load(min(c + 2, chunks - 1), even);
        step(c + 1, odd);
    }
    __syncthreads();
    store_o(chunks - 1);
#pragma unroll
    for (int j = 0; j < NB; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int d = 16 * (wave * NB + j) + 4 * q + i;
            if (d < D && col < D) state[(size_t)d * D + col] = S[j][i];
        }
}

// the head's norm and the output gate over the chunk form's outputs: one wave per (row, head)
template <class E>
__global__ void __launch_bounds__(256) k_delta_out(const DeltaArgs a, int row0) {
    typedef typename E::type T;
    const size_t m = row0 + blockIdx.x;
    const int head = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (head >= a.H) return;
    constexpr int R = DELTA_MAX_DIM / 64;
    const float *o = a.o + (m * a.H + head) * a.D8;
    float v[R], ss = 0.0f;
#pragma unroll
    for (int r = 0; r < R; ++r) v[r] = 64 * r + lane < a.D ? o[64 * r + lane] : 0.0f, ss = fmaf(v[r], v[r], ss);
    const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)a.D + a.eps);
    const int at = 3 * a.H * a.D8 + head * a.D8;
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int d = 64 * r + lane;
        if (d >= a.D) break;
        const float g = E::load((const T *)a.raw + m * a.ld + at + d) + (a.bias ? BF16::to_f32(a.bias[at + d]) : 0.0f);
        ((T *)a.out)[m * a.ld_out + head * a.D8 + d] = E::pack(v[r] * inv * a.o_norm[head * a.D + d] / (1.0f + expf(-g)));
    }
}

size_t delta_prep_lds(int NB, int R8) {
    const int R32 = (R8 + 31) & ~31;
    const size_t vec = (size_t)DC * (64 * NB + 4) * 4, low = (size_t)DC * (R32 + 8) * 4;  // (fp32, or bf16 halves)
    return vec + (5 * DC * 20 + DC + 64 * NB) * 4 + std::max(4 * vec, low);
}

template <class E, int NB>
int delta_chunks_nb(const DeltaArgs &a, int chunks, int row0, int rows, hipStream_t st) {
    const size_t lds = delta_prep_lds(NB, a.R8);
    PIE_REQUIRE(lds <= 160 * 1024, PIE_E_SHAPE, "delta rule: head and decay rank too large together");
    static bool raised = false;
    if (!raised) {
        PIE_HIP_TRY(hipFuncSetAttribute((const void *)k_delta_prep<E, NB>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024));
        raised = true;
    }
    hipLaunchKernelGGL((k_delta_prep<E, NB>), dim3((unsigned)chunks, (unsigned)a.H), dim3(256), lds, st, a);
    PIE_LAUNCH_CHECK();
    hipLaunchKernelGGL((k_delta_scan<E, NB>), dim3((unsigned)(a.H * dr_blocks(a.D)), (unsigned)a.n_runs), dim3(256), 0, st, a);
    PIE_LAUNCH_CHECK();
    hipLaunchKernelGGL(k_delta_out<E>, dim3((unsigned)rows, (unsigned)((a.H + 3) / 4)), dim3(256), 0, st, a, row0);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}
template <class E>
int delta_chunks_go(const DeltaArgs &a, int chunks, int row0, int rows, hipStream_t st) {
    if (a.D <= 64) return delta_chunks_nb<E, 1>(a, chunks, row0, rows, st);
    if (a.D <= 128) return delta_chunks_nb<E, 2>(a, chunks, row0, rows, st);
    if (a.D <= 192) return delta_chunks_nb<E, 3>(a, chunks, row0, rows, st);
    return delta_chunks_nb<E, 4>(a, chunks, row0, rows, st);
}

template <class E>
int delta_step_go(const DeltaArgs &a, hipStream_t st) {
    const dim3 grid((unsigned)a.n_runs, (unsigned)a.H);
#define DS_GO(CP_, NT_) hipLaunchKernelGGL((k_delta_step<E, CP_, NT_>), grid, dim3(NT_), 0, st, a)
    if (a.D <= 16) DS_GO(16, 128);
    else if (a.D <= 32) DS_GO(32, 256);
    else if (a.D <= 64) DS_GO(64, 256);
    else if (a.D <= 128) DS_GO(128, 512);
    else DS_GO(256, 1024);
#undef DS_GO
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

}  // namespace

int delta_chunks(int n_rows) { return (n_rows + DC - 1) / DC; }
size_t delta_ws_floats(int chunks, int H, int D) { return (size_t)chunks * H * dr_chunk_floats(D); }

static int delta_check(const DeltaArgs &a) {
    PIE_REQUIRE(a.D > 0 && a.D <= DELTA_MAX_DIM && a.rank > 0 && a.rank <= DELTA_MAX_RANK && a.H > 0 && a.H <= 65535, PIE_E_SHAPE,
                "delta rule: heads of at most 256 channels, decay rank of at most 1024");
    PIE_REQUIRE(a.slots && a.state && a.n_slots > 0, PIE_E_ARG, "delta rule: no state slots");
    return PIE_OK;
}

int delta_step_launch(int dtype, const DeltaArgs &a, hipStream_t st) {
    if (a.n_runs <= 0) return PIE_OK;
    if (const int rc = delta_check(a)) return rc;
    return dtype == PIE_F32 ? delta_step_go<ElemF32>(a, st) : delta_step_go<ElemBF16>(a, st);
}

int delta_chunks_launch(int dtype, const DeltaArgs &a, int chunks, int row0, int rows, hipStream_t st) {
    if (a.n_runs <= 0) return PIE_OK;
    if (const int rc = delta_check(a)) return rc;
    PIE_REQUIRE(a.ws && a.o && chunks > 0 && a.n_runs <= 65535, PIE_E_ARG, "delta rule: the chunk form needs its workspace");
    return dtype == PIE_F32 ? delta_chunks_go<ElemF32>(a, chunks, row0, rows, st) : delta_chunks_go<ElemBF16>(a, chunks, row0, rows, st);
}
