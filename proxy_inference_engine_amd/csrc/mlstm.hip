// mlstm.hip -- the matrix memory of xLSTM (PIE_MIXER_MLSTM): per head a state S [key][value column], a vector n [key] and a running maximum m, all fp32, with
//   i = cap tanh((.) / cap),  f = log sigmoid(cap tanh((.) / cap)),  m_t = max(f + m_(t-1), i)            (m starts at 0)
//   S_t = e^(f + m_(t-1) - m_t) S_(t-1) + e^(i - m_t) k v^T,  n_t likewise with k alone,  o_t = S_t^T q / (max(|n_t . q|, e^(-m_t)) + den_eps).
// Both forms leave the sums and what they are divided by; the head's norm and the output gate follow (head_out.hip).
//
// A head's columns are independent of each other but for m, which is the same for all: every block of 16 columns keeps its own copy of it (and one more goes
// with n), so that no workgroup writes a number that another one still reads.
//
// Step form (decoded tokens, short runs, fp32 stacks): a workgroup per (run, head, 32 columns), the state in registers; the first block of a head also has n.
//
// Chunk form, 64 tokens at a time.  With b_t the sum of f inside the chunk, c_t = max over s <= t of (b_t - b_s + i_s), M and S in front of the chunk,
//   m_t = max(M + b_t, c_t),   sums_t = e^(M + b_t - m_t) S^T q_t + e^(c_t - m_t) sum_{s <= t} P_ts v_s,   P_ts = e^(b_t - b_s + i_s - c_t) q_t . k_s
//   S <- e^(M + b_L - m_L) S + e^(c_L - m_L) sum_s e^(b_L - b_s + i_s - c_L) k_s v_s^T
// where no exponent is above zero.  One launch (all chunks of all heads in parallel) makes b, c, P and the key weights, and leaves q, k^T, v and P in matrix operand order; one
// walks the chunks, a workgroup per head and 16 value columns, whose four waves split the key channels of S.  n is chained by a launch of its own (its additions are known
// beforehand: k summed with its weights), and the denominators follow from it, all chunks in parallel.
// q, k and v are bf16 numbers, so their products are exact in fp32; what meets them as an operand is fp32 split into bf16 parts: the weighted values that enter the
// state in three (24 bits), P and the state where it is read in two.
#include "mfma_store.hpp"  // w4m_pack
#include "stack_types.hpp"

typedef __attribute__((ext_vector_type(4))) float ml_f32x4;
typedef __attribute__((ext_vector_type(8))) __bf16 ml_bf16x8;

namespace {

constexpr int ML = 64;      // tokens of a chunk
constexpr int ML_COLS = 32; // value columns of a step workgroup
constexpr float ML_NEG = -1e30f;

__host__ __device__ __forceinline__ int ml_up4(int n) { return (n + 3) & ~3; }
__host__ __device__ __forceinline__ int ml_blocks(int V) { return (V + 15) / 16; }
// S [H][D][V4], n [H][D4], m [H][blocks + 1]
struct MlState {
    float *S, *n, *m;
};
__device__ __forceinline__ MlState ml_state(const MlstmArgs &a, const RowRun &run, int head) {
    float *p = recurrent_state(a.r, run);
    const int V4 = ml_up4(a.V), D4 = ml_up4(a.D);
    return {p + (size_t)head * a.D * V4, p + (size_t)a.H * a.D * V4 + head * D4, p + (size_t)a.H * a.D * V4 + a.H * D4 + head * (ml_blocks(a.V) + 1)};
}

template <class T>
__device__ __forceinline__ float ml_load(const T *p) {
    if constexpr (sizeof(T) == 4) return *p;
    else return BF16::to_f32(*p);
}
// tanh and log sigmoid of the capped gates, a few units in the last place (the library's in fp32 stacks)
template <bool F32>
__device__ __forceinline__ float ml_cap(float z, float cap) { return cap * (F32 ? tanhf(z / cap) : fast_tanh(z / cap)); }
template <bool F32>
__device__ __forceinline__ float ml_log_sigmoid(float z) { return fminf(z, 0.0f) - log1pf(F32 ? expf(-fabsf(z)) : __builtin_amdgcn_exp2f(-fabsf(z) * STACK_LOG2E)); }
struct MlGates {
    float i, f;
};
template <class T>
__device__ __forceinline__ MlGates ml_gates(const MlstmArgs &a, size_t m, int head) {
    constexpr bool F32 = sizeof(T) == 4;
    const T *g = (const T *)a.r.raw + m * a.r.ld + 2 * a.H * a.D8 + 2 * a.H * a.V8 + head;
    return {ml_cap<F32>(ml_load(g) + a.gate_bias[head], a.cap), ml_log_sigmoid<F32>(ml_cap<F32>(ml_load(g + a.H8) + a.gate_bias[a.H + head], a.cap))};
}

// ---------------------------------------------------------------- step form
__device__ __forceinline__ float ml_sum8(float v) { return xor32_sum(xor16_sum(v + ror8(v))); }  // over the wave's lanes with the same lane % 8

// RPT: key channels per thread (32 RPT >= D)
template <class E, int RPT>
__global__ void __launch_bounds__(256) k_mlstm_step(const MlstmArgs a) {
    typedef typename E::type T;
    __shared__ __attribute__((aligned(16))) float s_o[2][4][8][4], s_n[2][4];
    const int head = blockIdx.y, cq = threadIdx.x & 7, rg = threadIdx.x >> 3, wave = threadIdx.x >> 6, col = ML_COLS * blockIdx.x + 4 * cq;
    const RowRun run = a.r.runs[blockIdx.z];
    const int V4 = ml_up4(a.V), D = a.D;
    const MlState st = ml_state(a, run, head);
    const bool fresh = a.r.pos[run.row0] == 0, live = col < V4, has_n = blockIdx.x == 0;
    float4 S[RPT];
    float n[RPT];
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int r = rg + 32 * i;
        S[i] = !fresh && live && r < D ? *(const float4 *)(st.S + (size_t)r * V4 + col) : make_float4(0, 0, 0, 0);
        n[i] = has_n && !fresh && r < D ? st.n[r] : 0.0f;
    }
    float m = fresh ? 0.0f : st.m[2 * blockIdx.x];
    for (int j = 0; j < run.n_rows; ++j) {
        const size_t row = run.row0 + j;
        const T *x = (const T *)a.r.raw + row * a.r.ld + head * a.D8;
        float q[RPT], k[RPT], v[4];
#pragma unroll
        for (int i = 0; i < RPT; ++i) {
            const int r = min(rg + 32 * i, D - 1);
            q[i] = ml_load(x + r), k[i] = ml_load(x + a.H * a.D8 + r);
        }
        const T *xv = (const T *)a.r.raw + row * a.r.ld + 2 * a.H * a.D8 + head * a.V8;
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = ml_load(xv + min(col + i, a.V - 1));
        const MlGates g = ml_gates<T>(a, row, head);
        const float next = fmaxf(g.f + m, g.i), keep = expf(g.f + m - next), add = expf(g.i - next);
        m = next;
        float4 o = make_float4(0, 0, 0, 0);
        float nq = 0.0f;
#pragma unroll
        for (int i = 0; i < RPT; ++i) {
            const bool in = rg + 32 * i < D;
            const float ka = in ? add * k[i] : 0.0f, qs = in ? a.scale * q[i] : 0.0f;
            S[i] = make_float4(fmaf(keep, S[i].x, ka * v[0]), fmaf(keep, S[i].y, ka * v[1]), fmaf(keep, S[i].z, ka * v[2]), fmaf(keep, S[i].w, ka * v[3]));
            o.x = fmaf(qs, S[i].x, o.x), o.y = fmaf(qs, S[i].y, o.y), o.z = fmaf(qs, S[i].z, o.z), o.w = fmaf(qs, S[i].w, o.w);
            n[i] = fmaf(keep, n[i], ka);
            nq = fmaf(qs, n[i], nq);
        }
        o = make_float4(ml_sum8(o.x), ml_sum8(o.y), ml_sum8(o.z), ml_sum8(o.w)), nq = ml_sum8(nq);
        if ((threadIdx.x & 63) < 8) {
            *(float4 *)s_o[j & 1][wave][cq] = o;
            if (cq == 0) s_n[j & 1][wave] = nq;
        }
        __syncthreads();
        if (threadIdx.x < 8 && live) {
            const float4 p0 = *(const float4 *)s_o[j & 1][0][cq], p1 = *(const float4 *)s_o[j & 1][1][cq], p2 = *(const float4 *)s_o[j & 1][2][cq], p3 = *(const float4 *)s_o[j & 1][3][cq];
            *(float4 *)(a.o + (row * a.H + head) * a.V8 + col) =
                make_float4((p0.x + p1.x) + (p2.x + p3.x), (p0.y + p1.y) + (p2.y + p3.y), (p0.z + p1.z) + (p2.z + p3.z), (p0.w + p1.w) + (p2.w + p3.w));
        }
        if (has_n && threadIdx.x == 0) {
            const float z = (s_n[j & 1][0] + s_n[j & 1][1]) + (s_n[j & 1][2] + s_n[j & 1][3]);
            a.den[row * a.H + head] = fmaxf(fabsf(z), expf(-m)) + a.den_eps;
        }
    }
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int r = rg + 32 * i;
        if (r >= D) break;
        if (live) *(float4 *)(st.S + (size_t)r * V4 + col) = S[i];
        if (has_n && cq == 0) st.n[r] = n[i];
    }
    if (threadIdx.x < 2) {
        const int block = 2 * blockIdx.x + threadIdx.x, blocks = ml_blocks(a.V);
        if (block < blocks) st.m[block] = m;
        if (has_n && threadIdx.x == 0) st.m[blocks] = m;
    }
}

// ---------------------------------------------------------------- chunk form
__host__ __device__ __forceinline__ int ml_pairs(int D) { return (D + 31) / 32; }  // 32-channel steps of the keys
// per (chunk, head), bytes: q [4 row tiles][pairs] KiB; k^T [pairs][2][2 token steps] KiB; P [4 row tiles][2 token steps][hi, lo] KiB; b, c, key weights, sums of P's rows [64]
// fp32 each; v [16-column blocks][2 token steps] KiB; [32 pairs] fp32 k summed with its weights (once chained: n in front of the chunk) and the maximum in front of it
struct MlChunk {
    size_t k, p, s, v, n, bytes;  // where they begin
};
__host__ __device__ __forceinline__ MlChunk ml_chunk(int D, int V) {
    const size_t np = ml_pairs(D);
    const size_t n = np * 8192 + 17408 + (size_t)ml_blocks(V) * 2048;
    return {np * 4096, np * 8192, np * 8192 + 16384, np * 8192 + 17408, n, n + np * 128 + 128};
}

__device__ __forceinline__ ml_f32x4 ml_mfma(const uint4 &a, const uint4 &b, const ml_f32x4 &c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(ml_bf16x8, a), __builtin_bit_cast(ml_bf16x8, b), c, 0, 0, 0);
}
// two fp32 numbers -> their leading bf16 parts; what is left stays in (x, y)
__device__ __forceinline__ u32 ml_part(float &x, float &y) {
    const u32 w = w4m_pack<BF16>(x, y);
    x -= lo_f32<BF16>(w), y -= hi_f32<BF16>(w);
    return w;
}

constexpr int ML_VB = 4;  // 16-column blocks of v per wave
// One workgroup per (chunk, head), wave w owning the chunk's rows 16 w .. + 15; behind them (blockIdx.z > 0) the ones that turn v round.
__global__ void __launch_bounds__(256) k_mlstm_prep(const MlstmArgs a) {
    constexpr int LP = ML + 8, LV = 16 * ML_VB + 2;  // u16 per row of P's parts, and of what is turned round (odd dwords)
    __shared__ __attribute__((aligned(16))) u16 s_t[2 * ML * LP > 4 * ML * LV ? 2 * ML * LP : 4 * ML * LV];
    __shared__ __attribute__((aligned(16))) float s_b[ML], s_c[ML], s_g[ML], s_w[ML];
    const int head = blockIdx.x, lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), n16 = lane & 15, q4 = lane >> 4;
    const RowChunk c = row_chunk(a.r.runs, a.r.n_runs, blockIdx.y, ML);
    if (c.n <= 0) return;
    const int np = ml_pairs(a.D), ld = a.r.ld;
    const MlChunk at = ml_chunk(a.D, a.V);
    char *ws = (char *)a.r.ws + ((size_t)blockIdx.y * a.H + head) * at.bytes;
    float *o_s = (float *)(ws + at.s);
    const u16 *raw = (const u16 *)a.r.raw + (size_t)c.row0 * ld + head * a.D8, *rk = raw + a.H * a.D8;
    auto piece = [&](const u16 *p, int row, int d) { return d < a.D8 ? *(const uint4 *)(p + (size_t)min(row, c.n - 1) * ld + d) : make_uint4(0, 0, 0, 0); };

    if (blockIdx.z) {
        // v: operand (block b, token step s) has column 16 b + n16 in lane n16, tokens 32 s + 8 q4 ..; a wave turns 64 columns of the 64 rows round in LDS
        const int b0 = ((int)blockIdx.z - 1) * 4 * ML_VB + wave * ML_VB, col = 16 * b0 + 8 * (lane & 7);
        if (b0 >= ml_blocks(a.V)) return;
        const u16 *rv = (const u16 *)a.r.raw + (size_t)c.row0 * ld + 2 * a.H * a.D8 + head * a.V8 + col;
        uint4 x[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) x[i] = col < a.V8 ? *(const uint4 *)(rv + (size_t)min(8 * i + (lane >> 3), c.n - 1) * ld) : make_uint4(0, 0, 0, 0);
        u16 *t = s_t + wave * ML * LV;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            u32 *d = (u32 *)(t + (8 * i + (lane >> 3)) * LV + 8 * (lane & 7));
            d[0] = x[i].x, d[1] = x[i].y, d[2] = x[i].z, d[3] = x[i].w;
        }
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // (a wave reads what it wrote)
#pragma unroll
        for (int j = 0; j < ML_VB; ++j) {
            if (b0 + j >= ml_blocks(a.V)) continue;
#pragma unroll
            for (int s = 0; s < 2; ++s) {
                u32 w[4];
#pragma unroll
                for (int i = 0; i < 4; ++i) w[i] = t[(32 * s + 8 * q4 + 2 * i) * LV + 16 * j + n16] | (u32)t[(32 * s + 8 * q4 + 2 * i + 1) * LV + 16 * j + n16] << 16;
                *(uint4 *)(ws + at.v + (size_t)(2 * (b0 + j) + s) * 1024 + lane * 16) = make_uint4(w[0], w[1], w[2], w[3]);
            }
        }
        return;
    }
    if (wave == 0) {  // lane: token
        MlGates g = {ML_NEG, 0.0f};
        if (lane < c.n) g = ml_gates<u16>(a, c.row0 + lane, head);
        float b = g.f, m = g.i;
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) {  // (a, max) pairs: (a1, m1) then (a2, m2) = (a1 + a2, max(m1 + a2, m2))
            const float b1 = __shfl_up(b, o, 64), m1 = __shfl_up(m, o, 64);
            if (lane >= o) m = fmaxf(m1 + b, m), b += b1;
        }
        s_b[lane] = b, s_c[lane] = m, s_g[lane] = g.i;
        const float bl = __shfl(b, 63, 64), cl = __shfl(m, 63, 64);
        const float w = lane < c.n ? stack_exp<false>(bl - b + g.i - cl) : 0.0f;
        s_w[lane] = w, o_s[lane] = b, o_s[ML + lane] = m, o_s[2 * ML + lane] = w;
    }
    ml_f32x4 acc[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) acc[t] = (ml_f32x4){0.0f, 0.0f, 0.0f, 0.0f};
    for (int p = 0; p < np; ++p) {
        const uint4 qv = piece(raw, 16 * wave + n16, 32 * p + 8 * q4);
        *(uint4 *)(ws + ((size_t)wave * np + p) * 1024 + lane * 16) = qv;
#pragma unroll
        for (int t = 0; t < 4; ++t)
            if (t <= wave) acc[t] = ml_mfma(qv, piece(rk, 16 * t + n16, 32 * p + 8 * q4), acc[t]);
    }
    __syncthreads();
    // k^T: operand (pair p, half e, token step s) has channel 32 p + 8 (n16 / 4) + 4 e + n16 % 4 in lane n16, tokens 32 s + 8 q4 ..
    for (int i = wave; i < 2 * np; i += 4) {
        const int d = 32 * (i >> 1) + 8 * (n16 >> 2) + 4 * (i & 1) + (n16 & 3);
        u16 v[2][8];
#pragma unroll
        for (int s = 0; s < 2; ++s)
#pragma unroll
            for (int k = 0; k < 8; ++k) v[s][k] = rk[(size_t)min(32 * s + 8 * q4 + k, c.n - 1) * ld + min(d, a.D8 - 1)];
        float sum = 0.0f;
#pragma unroll
        for (int s = 0; s < 2; ++s) {
#pragma unroll
            for (int k = 0; k < 8; ++k) sum = fmaf(BF16::to_f32(v[s][k]), s_w[32 * s + 8 * q4 + k], sum);
            uint4 w = make_uint4(v[s][0] | (u32)v[s][1] << 16, v[s][2] | (u32)v[s][3] << 16, v[s][4] | (u32)v[s][5] << 16, v[s][6] | (u32)v[s][7] << 16);
            if (d >= a.D) w = make_uint4(0, 0, 0, 0);
            *(uint4 *)(ws + at.k + (size_t)(2 * i + s) * 1024 + lane * 16) = w;
        }
        sum = xor32_sum(xor16_sum(sum));
        if (q4 == 0) ((float *)(ws + at.n))[d] = d < a.D ? sum : 0.0f;
    }
    // rows 16 wave + 4 q4 + i, columns 16 t + n16
    float rows[4] = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int row = 16 * wave + 4 * q4 + i, s = 16 * t + n16;
            float x = s <= row && row < c.n ? a.scale * acc[t][i] * stack_exp<false>(s_b[row] - s_b[s] + s_g[s] - s_c[row]) : 0.0f, y = 0.0f;
            rows[i] += x;
            const u16 hi = BF16::from_f32(x);
            y = x - BF16::to_f32(hi);
            s_t[row * LP + s] = hi, s_t[(ML + row) * LP + s] = BF16::from_f32(y);
        }
#pragma unroll
    for (int i = 0; i < 4; ++i) rows[i] = lanes16_sum(rows[i]);
    if (n16 == 0) *(ml_f32x4 *)(o_s + 3 * ML + 16 * wave + 4 * q4) = (ml_f32x4){rows[0], rows[1], rows[2], rows[3]};
    // (a wave reads the rows it wrote)
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    char *o_p = ws + at.p + (size_t)wave * 4096;
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
        for (int k = 0; k < 2; ++k) *(uint4 *)(o_p + (s * 2 + k) * 1024 + lane * 16) = *(const uint4 *)&s_t[(ML * k + 16 * wave + n16) * LP + 32 * s + 8 * q4];
}

// n and the maximum in front of every chunk (a thread per channel), then the denominators of a chunk's rows
__global__ void __launch_bounds__(MLSTM_CHUNK_MAX_DIM) k_mlstm_chain(const MlstmArgs a) {
    const int head = blockIdx.x, d = threadIdx.x, np32 = 32 * ml_pairs(a.D);
    const RowRun run = a.r.runs[blockIdx.y];
    int chunk0 = 0;
    for (int r = 0; r < (int)blockIdx.y; ++r) chunk0 += (a.r.runs[r].n_rows + ML - 1) / ML;
    const int chunks = (run.n_rows + ML - 1) / ML;
    const MlState st = ml_state(a, run, head);
    const bool fresh = a.r.pos[run.row0] == 0;
    const MlChunk at = ml_chunk(a.D, a.V);
    const size_t step = at.bytes * a.H;
    char *ws = (char *)a.r.ws + ((size_t)chunk0 * a.H + head) * at.bytes;
    float n = !fresh && d < a.D ? st.n[d] : 0.0f, m = fresh ? 0.0f : st.m[ml_blocks(a.V)];
    const int dd = min(d, np32 - 1);
    constexpr int U = 16;  // chunks in flight
    for (int c0 = 0; c0 < chunks; c0 += U) {
        float k[U], b[U], c[U];
#pragma unroll
        for (int i = 0; i < U; ++i) {
            const char *p = ws + (size_t)min(c0 + i, chunks - 1) * step;
            k[i] = ((const float *)(p + at.n))[dd], b[i] = ((const float *)(p + at.s))[ML - 1], c[i] = ((const float *)(p + at.s))[2 * ML - 1];
        }
#pragma unroll
        for (int i = 0; i < U; ++i) {
            if (c0 + i >= chunks) continue;
            float *p = (float *)(ws + (size_t)(c0 + i) * step + at.n);
            if (d < np32) p[d] = n;
            if (d == 0) p[np32] = m;
            const float next = fmaxf(m + b[i], c[i]);
            n = fmaf(stack_exp<false>(m + b[i] - next), n, stack_exp<false>(c[i] - next) * k[i]), m = next;
        }
    }
    __syncthreads();  // (everyone has read the old maximum)
    if (d < a.D) st.n[d] = n;
    if (d == 0) st.m[ml_blocks(a.V)] = m;
}
// one workgroup per (chunk, head), a wave per row; NP: channel pairs per lane
template <int NP>
__global__ void __launch_bounds__(256) k_mlstm_den(const MlstmArgs a) {
    const int head = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const RowChunk c = row_chunk(a.r.runs, a.r.n_runs, blockIdx.y, ML);
    const MlChunk at = ml_chunk(a.D, a.V);
    const char *ws = (const char *)a.r.ws + ((size_t)blockIdx.y * a.H + head) * at.bytes;
    const float *n = (const float *)(ws + at.n), *s = (const float *)(ws + at.s);
    const int last = 32 * ml_pairs(a.D);
    const float m = n[last];
    float2 nv[NP];
#pragma unroll
    for (int p = 0; p < NP; ++p) {
        const int d = 2 * (lane + 64 * p);
        nv[p] = d < last ? *(const float2 *)(n + d) : make_float2(0, 0);  // (zeros past the channels)
    }
    constexpr int U = 8;  // rows of a wave in flight
    for (int t0 = wave * 16; t0 < wave * 16 + 16; t0 += U) {
        u32 q[U][NP];
#pragma unroll
        for (int i = 0; i < U; ++i)
#pragma unroll
            for (int p = 0; p < NP; ++p)
                q[i][p] = *(const u32 *)((const u16 *)a.r.raw + (size_t)(c.row0 + min(t0 + i, c.n - 1)) * a.r.ld + head * a.D8 + min(2 * (lane + 64 * p), a.D8 - 2));
#pragma unroll
        for (int i = 0; i < U; ++i) {
            if (t0 + i >= c.n) continue;
            float dot = 0.0f;
#pragma unroll
            for (int p = 0; p < NP; ++p) dot = fmaf(lo_f32<BF16>(q[i][p]), nv[p].x, fmaf(hi_f32<BF16>(q[i][p]), nv[p].y, dot));
            dot = lanes_sum(dot);
            const float b = s[t0 + i], cc = s[ML + t0 + i], mt = fmaxf(m + b, cc);
            const float nq = fmaf(a.scale * stack_exp<false>(m + b - mt), dot, stack_exp<false>(cc - mt) * s[3 * ML + t0 + i]);
            if (lane == 0) a.den[(size_t)(c.row0 + t0 + i) * a.H + head] = fmaxf(fabsf(nq), stack_exp<false>(-mt)) + a.den_eps;
        }
    }
}

// NPW: 32-channel pairs per wave (D <= 128 NPW).  A chunk's operands are loaded where the previous chunk's have just been used, out of the L2: a head's workgroups share
// the reading of the chunk behind that from further away, a line per thread (into LDS that nobody reads).
template <int NPW>
__global__ void __launch_bounds__(256, 1) k_mlstm_scan(const MlstmArgs a) {
    __shared__ __attribute__((aligned(16))) ml_f32x4 s_o[2][4][4][64];
    __shared__ __attribute__((aligned(1024))) char s_warm[1024];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), n16 = lane & 15, q4 = lane >> 4;
    const int head = (int)blockIdx.x % a.H, cb = (int)blockIdx.x / a.H, V4 = ml_up4(a.V), D = a.D, np = ml_pairs(D);  // (head fastest: a head's columns share an L2 where H is a multiple of 8)
    const RowRun run = a.r.runs[blockIdx.y];
    int chunk0 = 0;
    for (int r = 0; r < (int)blockIdx.y; ++r) chunk0 += (a.r.runs[r].n_rows + ML - 1) / ML;
    const int chunks = (run.n_rows + ML - 1) / ML, col = 16 * cb + n16;
    const MlState st = ml_state(a, run, head);
    const bool fresh = a.r.pos[run.row0] == 0;
    // half e of pair P: register i <-> channel 32 P + 8 q4 + 4 e + i, column n16
    ml_f32x4 S[NPW][2];
    auto place = [&](int j, int e, int i) -> float * {
        const int d = 32 * (wave * NPW + j) + 8 * q4 + 4 * e + i;
        if (d >= D) return nullptr;
        return col < a.V ? st.S + (size_t)d * V4 + col : nullptr;
    };
#pragma unroll
    for (int j = 0; j < NPW; ++j)
#pragma unroll
        for (int e = 0; e < 2; ++e)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const float *p = place(j, e, i);
                S[j][e][i] = !fresh && p ? *p : 0.0f;
            }
    float m = fresh ? 0.0f : st.m[cb];
    const MlChunk place_of = ml_chunk(D, a.V);
    const size_t step = place_of.bytes * a.H;
    const char *ws0 = (const char *)a.r.ws + ((size_t)chunk0 * a.H + head) * place_of.bytes;
    uint4 q[4][NPW], k[NPW][2][2], p[2][2];
    uint4 v[2];
    ml_f32x4 w[2][2], nb, nc;  // key weights of the lane's tokens; b and c of its output rows
    float nbl, ncl;
    auto load_q = [&](int ch) {
        const char *ws = ws0 + (size_t)min(ch, chunks - 1) * step + lane * 16;
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int j = 0; j < NPW; ++j) q[t][j] = *(const uint4 *)(ws + ((size_t)t * np + min(wave * NPW + j, np - 1)) * 1024);
    };
    auto load_k = [&](int ch) {
        const char *ws = ws0 + (size_t)min(ch, chunks - 1) * step + place_of.k + lane * 16;
#pragma unroll
        for (int j = 0; j < NPW; ++j)
#pragma unroll
            for (int e = 0; e < 2; ++e)
#pragma unroll
                for (int s = 0; s < 2; ++s) k[j][e][s] = *(const uint4 *)(ws + (size_t)(4 * min(wave * NPW + j, np - 1) + 2 * e + s) * 1024);
    };
    auto load_pv = [&](int ch) {
        const char *ws = ws0 + (size_t)min(ch, chunks - 1) * step + lane * 16;
#pragma unroll
        for (int s = 0; s < 2; ++s) {
#pragma unroll
            for (int h = 0; h < 2; ++h) p[s][h] = *(const uint4 *)(ws + place_of.p + wave * 4096 + (s * 2 + h) * 1024);
            v[s] = *(const uint4 *)(ws + place_of.v + (size_t)(2 * cb + s) * 1024);
#pragma unroll
            for (int h = 0; h < 2; ++h) w[s][h] = *(const ml_f32x4 *)((const float *)(ws - lane * 16 + place_of.s) + 2 * ML + 32 * s + 8 * q4 + 4 * h);
        }
    };
    auto load_scalars = [&](int ch) {
        const float *sc = (const float *)(ws0 + (size_t)min(ch, chunks - 1) * step + place_of.s);
        nb = *(const ml_f32x4 *)(sc + 16 * wave + 4 * q4), nc = *(const ml_f32x4 *)(sc + ML + 16 * wave + 4 * q4), nbl = sc[ML - 1], ncl = sc[2 * ML - 1];
    };
    const unsigned line = (unsigned)min((cb * 256 + (int)threadIdx.x) * 128, (int)place_of.bytes - 4) & ~3u, warm_lds = (unsigned)(size_t)(__attribute__((address_space(3))) void *)s_warm + 256u * wave;
    auto warm = [&](int ch) {
        const unsigned long long v = (unsigned long long)(uintptr_t)(ws0 + (size_t)min(ch, chunks - 1) * step);
        const unsigned long long src =
            (unsigned long long)(unsigned)__builtin_amdgcn_readfirstlane((int)(unsigned)v) | ((unsigned long long)(unsigned)__builtin_amdgcn_readfirstlane((int)(unsigned)(v >> 32)) << 32);
        unsigned keep;
        asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %3\n\ts_nop 0\n\tglobal_load_lds_dword %1, %2\n\ts_mov_b32 m0, %0" : "=&s"(keep) : "v"(line), "s"(src), "s"(warm_lds) : "memory");
    };
    load_scalars(0), load_q(0), load_pv(0), load_k(0), warm(1);
    const ml_f32x4 zero = {0.0f, 0.0f, 0.0f, 0.0f};
    for (int ch = 0; ch < chunks; ++ch) {
        const ml_f32x4 cbv = nb, ccv = nc;
        const float bl = nbl, cl = ncl;
        load_scalars(ch + 1);
        const float next = fmaxf(m + bl, cl), keep = stack_exp<false>(m + bl - next), add = stack_exp<false>(cl - next);
        // S^T q of the chunk's 64 rows: the wave's channels
        ml_f32x4 acc[4] = {zero, zero, zero, zero};
#pragma unroll
        for (int j = 0; j < NPW; ++j) {
            float f[8];
            u32 hi[4], lo[4];
#pragma unroll
            for (int i = 0; i < 8; ++i) f[i] = S[j][i >> 2][i & 3];
#pragma unroll
            for (int i = 0; i < 4; ++i) hi[i] = ml_part(f[2 * i], f[2 * i + 1]), lo[i] = w4m_pack<BF16>(f[2 * i], f[2 * i + 1]);
            const uint4 h = make_uint4(hi[0], hi[1], hi[2], hi[3]), l = make_uint4(lo[0], lo[1], lo[2], lo[3]);
#pragma unroll
            for (int t = 0; t < 4; ++t) acc[t] = ml_mfma(q[t][j], h, acc[t]);
#pragma unroll
            for (int t = 0; t < 4; ++t) acc[t] = ml_mfma(q[t][j], l, acc[t]);
        }
        load_q(ch + 1);
#pragma unroll
        for (int t = 0; t < 4; ++t) s_o[ch & 1][wave][t][lane] = acc[t];
        // the wave's own rows among themselves
        ml_f32x4 own = zero;
        float f[2][8];
#pragma unroll
        for (int s = 0; s < 2; ++s) {
            const u32 x[4] = {v[s].x, v[s].y, v[s].z, v[s].w};
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                f[s][2 * i] = lo_f32<BF16>(x[i]) * (add * w[s][i >> 1][2 * (i & 1)]);
                f[s][2 * i + 1] = hi_f32<BF16>(x[i]) * (add * w[s][i >> 1][2 * (i & 1) + 1]);
            }
            own = ml_mfma(p[s][0], v[s], own), own = ml_mfma(p[s][1], v[s], own);
        }
        load_pv(ch + 1);
        // the state behind the chunk: values times their key weights, in three parts
#pragma unroll
        for (int j = 0; j < NPW; ++j)
#pragma unroll
            for (int e = 0; e < 2; ++e) S[j][e] *= keep;
#pragma unroll
        for (int s = 0; s < 2; ++s)
#pragma unroll
            for (int h = 0; h < 3; ++h) {
                u32 x[4];
#pragma unroll
                for (int i = 0; i < 4; ++i) x[i] = h < 2 ? ml_part(f[s][2 * i], f[s][2 * i + 1]) : w4m_pack<BF16>(f[s][2 * i], f[s][2 * i + 1]);
                const uint4 part = make_uint4(x[0], x[1], x[2], x[3]);
#pragma unroll
                for (int j = 0; j < NPW; ++j)
#pragma unroll
                    for (int e = 0; e < 2; ++e) S[j][e] = ml_mfma(k[j][e][s], part, S[j][e]);
            }
        load_k(ch + 1);
        warm(ch + 2);
#pragma unroll
        for (int j = 0; j < NPW; ++j)
            if (wave * NPW + j >= np) S[j][0] = S[j][1] = zero;  // (channels that do not exist saw another pair's keys)
        asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");  // (LDS only: the next chunk's loads stay in flight)
        const ml_f32x4 all = (s_o[ch & 1][0][wave][lane] + s_o[ch & 1][1][wave][lane]) + (s_o[ch & 1][2][wave][lane] + s_o[ch & 1][3][wave][lane]);
        float o[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const float mt = fmaxf(m + cbv[i], ccv[i]);
            o[i] = fmaf(a.scale * stack_exp<false>(m + cbv[i] - mt), all[i], stack_exp<false>(ccv[i] - mt) * own[i]);
        }
        const int t0 = ML * ch + 16 * wave + 4 * q4;
        const size_t at = ((size_t)run.row0 + t0) * a.H + head;
        if (col < a.V) {
            float *dst = a.o + at * a.V8 + col;
            const int row = a.H * a.V8;
            if (ML * (ch + 1) <= run.n_rows)
#pragma unroll
                for (int i = 0; i < 4; ++i) dst[i * row] = o[i];
            else
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    if (t0 + i < run.n_rows) dst[i * row] = o[i];
        }
        m = next;
    }
#pragma unroll
    for (int j = 0; j < NPW; ++j)
#pragma unroll
        for (int e = 0; e < 2; ++e)
#pragma unroll
            for (int i = 0; i < 4; ++i)
                if (float *x = place(j, e, i)) *x = S[j][e][i];
    if (threadIdx.x == 0) st.m[cb] = m;
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // (what was read ahead: LDS is handed on when the workgroup ends)
}

int mlstm_check(const MlstmArgs &a) {
    PIE_REQUIRE(a.H > 0 && a.H <= 65535 && a.D > 0 && a.D <= MLSTM_MAX_DIM && a.V > 0 && a.cap > 0, PIE_E_SHAPE, "mLSTM: keys of at most 1024 channels per head");
    PIE_REQUIRE(a.r.slots && a.r.state && a.r.n_slots > 0 && a.r.slot_floats % 4 == 0 && a.gate_bias && a.o && a.den && a.r.n_runs <= 65535, PIE_E_ARG, "mLSTM: no state slots or workspace");
    return PIE_OK;
}

template <class E>
void mlstm_step_go(const MlstmArgs &a, hipStream_t st) {
    const dim3 grid((unsigned)((a.V + ML_COLS - 1) / ML_COLS), (unsigned)a.H, (unsigned)a.r.n_runs);
#define ST_GO(N_) hipLaunchKernelGGL((k_mlstm_step<E, N_>), grid, dim3(256), 0, st, a)
    if (a.D <= 32) ST_GO(1);
    else if (a.D <= 64) ST_GO(2);
    else if (a.D <= 128) ST_GO(4);
    else if (a.D <= 256) ST_GO(8);
    else if (a.D <= 512) ST_GO(16);
    else ST_GO(32);
#undef ST_GO
}

}  // namespace

size_t mlstm_state_floats(int H, int D, int V) { return (size_t)H * D * ml_up4(V) + (size_t)H * ml_up4(D) + (size_t)H * (ml_blocks(V) + 1); }
int mlstm_chunks(int n_rows) { return (n_rows + ML - 1) / ML; }
size_t mlstm_ws_floats(int chunks, int H, int D, int V) { return (size_t)chunks * H * ml_chunk(D, V).bytes / 4; }

int mlstm_step_launch(int dtype, const MlstmArgs &a, hipStream_t st) {
    if (a.r.n_runs <= 0) return PIE_OK;
    if (const int rc = mlstm_check(a)) return rc;
    if (dtype == PIE_F32) mlstm_step_go<ElemF32>(a, st);
    else mlstm_step_go<ElemBF16>(a, st);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

int mlstm_chunks_launch(const MlstmArgs &a, int chunks, hipStream_t st) {
    if (a.r.n_runs <= 0) return PIE_OK;
    if (const int rc = mlstm_check(a)) return rc;
    PIE_REQUIRE(a.r.ws && chunks > 0 && chunks <= 65535 && a.D <= MLSTM_CHUNK_MAX_DIM, PIE_E_ARG, "mLSTM: the chunk form needs its workspace, and keys of at most 512 channels");
    hipLaunchKernelGGL(k_mlstm_prep, dim3((unsigned)a.H, (unsigned)chunks, (unsigned)(1 + (ml_blocks(a.V) + 4 * ML_VB - 1) / (4 * ML_VB))), dim3(256), 0, st, a);
    PIE_LAUNCH_CHECK();
    hipLaunchKernelGGL(k_mlstm_chain, dim3((unsigned)a.H, (unsigned)a.r.n_runs), dim3((unsigned)((32 * ml_pairs(a.D) + 63) / 64 * 64)), 0, st, a);
    PIE_LAUNCH_CHECK();
    const dim3 dg((unsigned)a.H, (unsigned)chunks);
    if (a.D <= 128) hipLaunchKernelGGL(k_mlstm_den<1>, dg, dim3(256), 0, st, a);
    else if (a.D <= 256) hipLaunchKernelGGL(k_mlstm_den<2>, dg, dim3(256), 0, st, a);
    else hipLaunchKernelGGL(k_mlstm_den<4>, dg, dim3(256), 0, st, a);
    PIE_LAUNCH_CHECK();
    const dim3 grid((unsigned)(a.H * ml_blocks(a.V)), (unsigned)a.r.n_runs);
    if (a.D <= 128) hipLaunchKernelGGL(k_mlstm_scan<1>, grid, dim3(256), 0, st, a);
    else if (a.D <= 256) hipLaunchKernelGGL(k_mlstm_scan<2>, grid, dim3(256), 0, st, a);
    else hipLaunchKernelGGL(k_mlstm_scan<4>, grid, dim3(256), 0, st, a);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}
