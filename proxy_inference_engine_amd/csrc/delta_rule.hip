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
// split the key channels of S (which stays in accumulators and is its own B operand); a third takes the heads' norm and gate.  W_16 is
// above exp(-16 decay_scale): the quotients are formed as W_t times 1 / W_i, which fp32 holds up to DELTA_MAX_DECAY.
#include <algorithm>

#include "stack_types.hpp"

typedef __attribute__((ext_vector_type(4))) float dr_f32x4;
typedef __attribute__((ext_vector_type(8))) __bf16 dr_bf16x8;

namespace {

constexpr int DC = 16;  // tokens of a chunk
constexpr size_t DELTA_SEGMENT_BYTES = 96u << 20;

__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }  // (loads and stores stay in flight)

// CP: power of two >= D; NT threads; AHEAD: few workgroups, where latency counts and registers do not
template <class E, int CP, int NT, bool AHEAD>
__global__ void __launch_bounds__(NT, AHEAD ? 1 : 4) k_delta_step(const DeltaArgs a) {
    typedef typename E::type T;
    constexpr int SL = NT / CP, RPT = CP / SL;  // channel slices; channels per thread
    static_assert(NT % CP == 0 && CP % SL == 0 && NT % 64 == 0, "slices");
    __shared__ __attribute__((aligned(16))) float s_r[CP], s_k[CP], s_v[CP], s_g[CP], s_a[CP], s_w[CP], s_low[DELTA_MAX_RANK], s_p[SL][CP], s_o[SL][CP], s_ss[NT / 64];
    const int run_i = blockIdx.x, head = blockIdx.y, D = a.D, lane = threadIdx.x & 63;
    const RowRun run = a.runs[run_i];
    const int col = threadIdx.x % CP, slice = threadIdx.x / CP, d0 = slice * RPT;
    const int seq = min(a.row_seq[run.row0], a.n_seqs - 1);
    const size_t slot = min((unsigned)a.slots[seq], (unsigned)a.n_slots - 1u);
    float *state = a.state + slot * a.slot_floats + (size_t)head * D * D;
    float S[RPT];
    const bool fresh = a.pos[run.row0] == 0;
#pragma unroll
    for (int i = 0; i < RPT; ++i) S[i] = !fresh && col < D && d0 + i < D ? state[(size_t)(d0 + i) * D + col] : 0.0f;
    const int HD8 = a.H * a.D8;
    // AHEAD: what all tokens share leaves together with the state -- the decay's weights (eight lanes per channel, the first WS pieces) and the head's norm
    constexpr int CPT = (CP + NT / 8 - 1) / (NT / 8), WS = 2;
    uint4 wd[AHEAD ? CPT : 1][WS];
    float db[AHEAD ? CPT : 1], o_norm = 0.0f;
    auto decay_weights = [&](int d, int i) { return *(const uint4 *)(a.w_decay + (size_t)(head * D + min(d, D - 1)) * a.R8 + min(i, a.R8 - 8)); };
    if constexpr (AHEAD) o_norm = a.o_norm[head * D + min((int)threadIdx.x, D - 1)];
#pragma unroll
    for (int c = 0; c < (AHEAD ? CPT : 0); ++c) {
        const int d = (threadIdx.x >> 3) + c * (NT / 8);
#pragma unroll
        for (int s = 0; s < WS; ++s) wd[c][s] = decay_weights(d, (threadIdx.x & 7) * 8 + 64 * s);
        db[c] = a.decay_bias[head * D + min(d, D - 1)];
    }

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
        lds_barrier();
        auto part = [&](float z, int i, const uint4 &w) {
            const float4 l0 = *(const float4 *)(s_low + i), l1 = *(const float4 *)(s_low + i + 4);
            z = fmaf(lo_f32<BF16>(w.x), l0.x, fmaf(hi_f32<BF16>(w.x), l0.y, fmaf(lo_f32<BF16>(w.y), l0.z, fmaf(hi_f32<BF16>(w.y), l0.w, z))));
            return fmaf(lo_f32<BF16>(w.z), l1.x, fmaf(hi_f32<BF16>(w.z), l1.y, fmaf(lo_f32<BF16>(w.w), l1.z, fmaf(hi_f32<BF16>(w.w), l1.w, z))));
        };
        auto put_decay = [&](int d, float z, float bias) {
            z = lanes8_sum(z);
            if ((threadIdx.x & 7) == 0 && d < CP) s_w[d] = d < D ? expf(-a.decay_scale / (1.0f + expf(-(z + bias)))) : 1.0f;
        };
        if constexpr (AHEAD)
#pragma unroll
            for (int c = 0; c < CPT; ++c) {
                const int d = (threadIdx.x >> 3) + c * (NT / 8);
                float z = 0.0f;
#pragma unroll
                for (int s = 0; s < WS; ++s)
                    if ((int)(threadIdx.x & 7) * 8 + 64 * s < a.R8) z = part(z, (threadIdx.x & 7) * 8 + 64 * s, wd[c][s]);
                for (int i = (threadIdx.x & 7) * 8 + 64 * WS; i < a.R8; i += 64) z = part(z, i, decay_weights(d, i));
                put_decay(d, z, db[c]);
            }
        else
#pragma unroll 1
            for (int d = threadIdx.x >> 3; d < CP; d += NT / 8) {
                float z = 0.0f;
                for (int i = (threadIdx.x & 7) * 8; i < a.R8; i += 64) z = part(z, i, decay_weights(d, i));
                put_decay(d, z, a.decay_bias[head * D + min(d, D - 1)]);
            }
        float ss = 0.0f;  // every wave: the key's length
        for (int d = lane; d < CP; d += 64) ss = fmaf(s_k[d], s_k[d], ss);
        const float unit = 1.0f / sqrtf(wave_sum(ss) + a.unit_eps);
        float p = 0.0f;
#pragma unroll
        for (int i = 0; i < RPT; ++i) p = fmaf(s_k[d0 + i], S[i], p);
        s_p[slice][col] = p * unit;
        lds_barrier();
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
        lds_barrier();
        if (threadIdx.x < (CP < 64 ? 64 : CP)) {  // whole waves
            o = 0.0f;
            if (threadIdx.x < CP)
#pragma unroll
                for (int i = 0; i < SL; ++i) o += s_o[i][col];
            const float sum = wave_sum(o * o);
            if (lane == 0) s_ss[threadIdx.x >> 6] = sum;
        }
        lds_barrier();
        if (threadIdx.x < D) {
            float sum = s_ss[0];
#pragma unroll
            for (int i = 1; i < (CP + 63) / 64; ++i) sum += s_ss[i];
            const float y = o * (1.0f / sqrtf(sum / (float)D + a.eps)) * (AHEAD ? o_norm : a.o_norm[head * D + threadIdx.x]) * s_g[threadIdx.x];
            ((T *)a.out)[m * a.ld_out + head * a.D8 + threadIdx.x] = E::pack(y);
        }
        lds_barrier();  // the channel vectors are written again
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

// One workgroup per (chunk, head).  A wave owns four tokens; its lanes own channel pairs.
// NB: 16-channel blocks per wave in the products (D <= 64 NB).  Dynamic LDS: see delta_prep_lds().
template <class E, int NB>
__global__ void __launch_bounds__(256) k_delta_prep(const DeltaArgs a) {
    typedef typename E::type T;
    constexpr bool F32 = sizeof(T) == 4;
    constexpr int LD = 64 * NB + 4, NP = (NB + 1) / 2, TP = DC / 4, LM = 20;  // NP: channel pairs per lane; TP: tokens per wave
    extern __shared__ __attribute__((aligned(16))) char lds[];
    float *s_l = (float *)lds, *s_m = s_l + DC * LD, *s_wc = s_m + 5 * DC * LM;  // log decays; A, B (transposed), A', B', T; W_16
    float *s_u = s_wc + 64 * NB, *s_r = s_u + DC * LD, *s_k = s_r + DC * LD, *s_a = s_k + DC * LD;
    // (the low-rank input of the decay lies where the channel vectors come later)
    const int D = a.D, nblk = dr_blocks(D), lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), n16 = lane & 15, q = lane >> 4;
    const int head = blockIdx.x, HD8 = a.H * a.D8;  // (head fastest: workgroups that run together read whole rows)
    const DeltaChunk c = dr_chunk(a, a.chunk_lo + (int)blockIdx.y);
    if (c.n <= 0) return;
    const int R32 = (a.R8 + 31) & ~31, LR = R32 + 8;
    u16 *s_hi = (u16 *)s_u, *s_lo = s_hi + DC * LR;
    float *s_low = s_u;
    struct Pair {
        float x, y;
    };
    auto pair_at = [&](const T *p) -> Pair {
        if constexpr (F32) return {((const float2 *)p)->x, ((const float2 *)p)->y};
        else {
            const u32 w = *(const u32 *)p;
            return {lo_f32<BF16>(w), hi_f32<BF16>(w)};
        }
    };
    auto bias_at = [&](int at) -> Pair {
        if (!a.bias) return {0.0f, 0.0f};
        const u32 w = *(const u32 *)(a.bias + at);
        return {lo_f32<BF16>(w), hi_f32<BF16>(w)};
    };
    // All loads without branches around them: they leave together, and what lies outside is dropped afterwards.
    const T *raw = (const T *)a.raw + (size_t)c.row0 * a.ld;
    constexpr int LN = 4;  // pairs of the low-rank input per thread that travel ahead (ranks up to 128): sixteen lanes per token
    const int tr = threadIdx.x >> 4, lr = 2 * (threadIdx.x & 15);
    Pair low[LN], lowb[LN];
#pragma unroll
    for (int j = 0; j < LN; ++j) {
        const int at = 5 * HD8 + min(lr + 32 * j, a.R8 - 2);
        low[j] = pair_at(raw + (size_t)min(tr, c.n - 1) * a.ld + at), lowb[j] = bias_at(at);
    }
    Pair xr[NP][TP], xk[NP][TP], xa[NP][TP], bx[NP][3];
#pragma unroll
    for (int p = 0; p < NP; ++p) {
        const int d = min(2 * (lane + 64 * p), a.D8 - 2) + head * a.D8;  // (heads are padded to a multiple of 8)
#pragma unroll
        for (int j = 0; j < TP; ++j) {
            const T *x = raw + (size_t)min(TP * wave + j, c.n - 1) * a.ld;
            xr[p][j] = pair_at(x + d), xk[p][j] = pair_at(x + HD8 + d), xa[p][j] = pair_at(x + 4 * HD8 + d);
        }
        bx[p][0] = bias_at(d), bx[p][1] = bias_at(HD8 + d), bx[p][2] = bias_at(4 * HD8 + d);
    }
    // the decay's weights (the first WS steps)
    constexpr int WS = 4;
    uint4 wd[F32 ? 1 : NB][WS];
    float db[NB];
    auto decay_weights = [&](int j, int s) {
        const int d = 16 * (wave * NB + j) + n16, at = 32 * s + 8 * q;
        const uint4 w = *(const uint4 *)(a.w_decay + (size_t)(head * D + min(d, D - 1)) * a.R8 + min(at, a.R8 - 8));
        return d < D && at < a.R8 ? w : make_uint4(0, 0, 0, 0);
    };
    if constexpr (!F32)
#pragma unroll
        for (int j = 0; j < NB; ++j) {
#pragma unroll
            for (int s = 0; s < WS; ++s) wd[j][s] = decay_weights(j, s);
            db[j] = a.decay_bias[head * D + min(16 * (wave * NB + j) + n16, D - 1)];
        }
    auto put_low = [&](int j, const Pair &v, const Pair &b) {
        auto f = [&](int i, float z) { return tr < c.n && i < a.rank ? F32 ? tanhf(z) : fast_tanh(z) : 0.0f; };
        const float x = f(j, v.x + b.x), y = f(j + 1, v.y + b.y);
        if constexpr (F32) s_low[tr * LR + j] = x, s_low[tr * LR + j + 1] = y;
        else {
            const u32 hi = pack2<BF16>(x, y);
            *(u32 *)(s_hi + tr * LR + j) = hi, *(u32 *)(s_lo + tr * LR + j) = pack2<BF16>(x - lo_f32<BF16>(hi), y - hi_f32<BF16>(hi));
        }
    };
#pragma unroll
    for (int j = 0; j < LN; ++j)
        if (32 * j < R32) put_low(lr + 32 * j, low[j], lowb[j]);
    for (int j = lr + 32 * LN; j < R32; j += 32) {
        const int at = 5 * HD8 + min(j, a.R8 - 2);
        put_low(j, pair_at(raw + (size_t)min(tr, c.n - 1) * a.ld + at), bias_at(at));
    }
    lds_barrier();
    auto log_decay = [&](int t, int d, float z) { s_l[t * LD + d] = t < c.n && d < D ? -a.decay_scale * stack_sigmoid<F32>(z) : 0.0f; };
    if constexpr (F32) {
        for (int i = threadIdx.x; i < DC * 16 * nblk; i += 256) {
            const int t = i / (16 * nblk), d = i % (16 * nblk);
            float z = 0.0f;
            if (d < D)
                for (int j = 0; j < a.rank; ++j) z = fmaf(s_low[t * LR + j], BF16::to_f32(a.w_decay[(size_t)(head * D + d) * a.R8 + j]), z);
            log_decay(t, d, z + a.decay_bias[head * D + min(d, D - 1)]);
        }
    } else {
#pragma unroll
        for (int j = 0; j < NB; ++j) {
            const int b = wave * NB + j, d = 16 * b + n16;
            if (b >= nblk) break;
            dr_f32x4 z = {0.0f, 0.0f, 0.0f, 0.0f};
            auto product = [&](int s, const uint4 &w) {
                const uint4 hi = *(const uint4 *)(s_hi + n16 * LR + 32 * s + 8 * q), lo = *(const uint4 *)(s_lo + n16 * LR + 32 * s + 8 * q);
                z = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(dr_bf16x8, hi), __builtin_bit_cast(dr_bf16x8, w), z, 0, 0, 0);
                z = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(dr_bf16x8, lo), __builtin_bit_cast(dr_bf16x8, w), z, 0, 0, 0);
            };
#pragma unroll
            for (int s = 0; s < WS; ++s)
                if (32 * s < R32) product(s, wd[j][s]);
            for (int s = WS; 32 * s < R32; ++s) product(s, decay_weights(j, s));
#pragma unroll
            for (int i = 0; i < 4; ++i) log_decay(4 * q + i, d, z[i] + db[j]);
        }
    }
    lds_barrier();  // the low-rank input has been read
    {
        float unit[TP];
#pragma unroll
        for (int j = 0; j < TP; ++j) {
            float ss = 0.0f;
#pragma unroll
            for (int p = 0; p < NP; ++p) {
                const int d = 2 * (lane + 64 * p);
                xk[p][j].x = d < D && TP * wave + j < c.n ? xk[p][j].x + bx[p][1].x : 0.0f, xk[p][j].y = d + 1 < D && TP * wave + j < c.n ? xk[p][j].y + bx[p][1].y : 0.0f;
                ss = fmaf(xk[p][j].x, xk[p][j].x, fmaf(xk[p][j].y, xk[p][j].y, ss));
            }
            unit[j] = 1.0f / sqrtf(wave_sum(ss) + a.unit_eps);
        }
#pragma unroll
        for (int p = 0; p < NP; ++p) {
            const int d = 2 * (lane + 64 * p);
            if (d >= 16 * nblk) break;
            float2 L = make_float2(0.0f, 0.0f);
            for (int t = 0; t < TP * wave; ++t) {
                const float2 l = *(const float2 *)(s_l + t * LD + d);
                L.x += l.x, L.y += l.y;
            }
            float2 before = make_float2(stack_exp<F32>(L.x), stack_exp<F32>(L.y));
#pragma unroll
            for (int j = 0; j < TP; ++j) {
                const int t = TP * wave + j, at = t * LD + d;
                const bool lx = t < c.n && d < D, ly = t < c.n && d + 1 < D;
                const float2 l = *(const float2 *)(s_l + at);
                L.x += l.x, L.y += l.y;
                const float2 e = make_float2(stack_exp<F32>(L.x), stack_exp<F32>(L.y)), back = make_float2(stack_exp<F32>(-L.x), stack_exp<F32>(-L.y));
                const float2 k = make_float2(xk[p][j].x, xk[p][j].y), u = make_float2(k.x * unit[j], k.y * unit[j]);
                *(float2 *)(s_u + at) = make_float2(u.x * before.x, u.y * before.y);
                *(float2 *)(s_r + at) = make_float2(lx ? (xr[p][j].x + bx[p][0].x) * e.x : 0.0f, ly ? (xr[p][j].y + bx[p][0].y) * e.y : 0.0f);
                *(float2 *)(s_k + at) = make_float2(k.x * back.x, k.y * back.y);
                *(float2 *)(s_a + at) = make_float2(stack_sigmoid<F32>(xa[p][j].x + bx[p][2].x) * u.x * back.x, stack_sigmoid<F32>(xa[p][j].y + bx[p][2].y) * u.y * back.y);
                before = e;
            }
            if (wave == 3) *(float2 *)(s_wc + d) = before;
        }
    }
    lds_barrier();
    {  // wave 0: A = U K^T, 1: B = U A^T, 2: A' = R K^T, 3: B' = R A^T
        const float *l = wave < 2 ? s_u : s_r, *r = wave & 1 ? s_a : s_k;
        dr_f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
        for (int b = 0; b < nblk; ++b) {
            const dr_f32x4 lv = *(const dr_f32x4 *)(l + n16 * LD + 16 * b + 4 * q), rv = *(const dr_f32x4 *)(r + n16 * LD + 16 * b + 4 * q);
#pragma unroll
            for (int i = 0; i < 4; ++i) acc = dr_mfma(lv[i], rv[i], acc);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) acc[i] = n16 < 4 * q + i + (wave >= 2) ? acc[i] : 0.0f;
        if (wave == 1) *(dr_f32x4 *)(s_m + (DC + n16) * LM + 4 * q) = acc;  // (B transposed)
        else
#pragma unroll
            for (int i = 0; i < 4; ++i) s_m[(wave * DC + 4 * q + i) * LM + n16] = acc[i];
    }
    lds_barrier();
    float *out = a.ws + ((size_t)blockIdx.y * a.H + head) * dr_chunk_floats(D);
    float *o_r = out + nblk * 256, *o_k = o_r + nblk * 256, *o_a = o_k + nblk * 256, *o_m = o_a + nblk * 256;
    float *s_t = s_m + 4 * DC * LM;
    if (wave == 0) {
        float tc[DC];  // column n16 of (I + B)^-1: forward substitution, column by column of B (stored transposed: rows are read whole)
#pragma unroll
        for (int t = 0; t < DC; ++t) tc[t] = t == n16 ? 1.0f : 0.0f;
#pragma unroll
        for (int i = 0; i < DC - 1; ++i)
#pragma unroll
            for (int t4 = i / 4; t4 < DC / 4; ++t4) {
                const dr_f32x4 col = *(const dr_f32x4 *)(s_m + (DC + i) * LM + 4 * t4);
#pragma unroll
                for (int k = 0; k < 4; ++k)
                    if (4 * t4 + k > i) tc[4 * t4 + k] = fmaf(-col[k], tc[i], tc[4 * t4 + k]);
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
    lds_barrier();
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

// A chunk's operands are further away than a chunk takes, so they travel through LDS by DMA, RING - 1 chunks ahead; every wave fetches, waits for and reads
// only its own.
template <class E, int NB>
struct ScanLds {
    static constexpr int DW = 16 * sizeof(typename E::type) / 4, VI = 16 * DW / 64;  // dwords of a token's 16 values; DMA instructions for the chunk's
    static constexpr int OPS = 4 * NB + 2 + VI;                                      // DMA instructions per wave and chunk
    static constexpr int WAVE = (4 * NB + 2) * 1024 + VI * 256, SLOT = 4 * WAVE;
    static constexpr int PB = NB <= 3 ? 2 : 1;  // buffers of the exchanges between the waves
    static constexpr int RING = 5 * SLOT <= 128 * 1024 ? 5 : 3 * SLOT <= 136 * 1024 ? 3 : 2;
};
template <class E, int NB>
__global__ void __launch_bounds__(256, 1) k_delta_scan(const DeltaArgs a) {
    typedef typename E::type T;
    typedef ScanLds<E, NB> L;
    __shared__ __attribute__((aligned(1024))) char s_ring[L::RING * L::SLOT];
    __shared__ dr_f32x4 s_p[L::PB][4][64], s_o[L::PB][4][64];
    const int D = a.D, nblk = dr_blocks(D), lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), n16 = lane & 15, q = lane >> 4;
    const int head = (int)blockIdx.x % a.H, cb = (int)blockIdx.x / a.H, col = 16 * cb + n16;  // (head fastest: the column blocks of a head share an L2 where H is a multiple of 8)
    const RowRun run = a.runs[blockIdx.y];
    int chunk0 = 0;
    for (int r = 0; r < (int)blockIdx.y; ++r) chunk0 += (a.runs[r].n_rows + DC - 1) / DC;
    const int c_lo = max(a.chunk_lo - chunk0, 0), c_hi = min(a.chunk_hi - chunk0, (run.n_rows + DC - 1) / DC);  // this launch's chunks of the run
    if (c_lo >= c_hi) return;
    const size_t slot = min((unsigned)a.slots[min(a.row_seq[run.row0], a.n_seqs - 1)], (unsigned)a.n_slots - 1u);
    float *state = a.state + slot * a.slot_floats + (size_t)head * D * D;
    const bool fresh = c_lo == 0 && a.pos[run.row0] == 0;
    dr_f32x4 S[NB];  // S[16 b + 4 q + i][col]
#pragma unroll
    for (int j = 0; j < NB; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int d = 16 * (wave * NB + j) + 4 * q + i;
            S[j][i] = !fresh && d < D && col < D ? state[(size_t)d * D + col] : 0.0f;
        }
    const size_t per = dr_chunk_floats(D);
    const float *ws = a.ws + ((ptrdiff_t)(chunk0 - a.chunk_lo) * a.H + head) * (ptrdiff_t)per;  // chunk c of the run at c * H * per
    const char *vp = (const char *)((const T *)a.raw + (size_t)run.row0 * a.ld + 2 * a.H * a.D8 + head * a.D8 + 16 * cb);
    const float vbias = a.bias ? BF16::to_f32(a.bias[2 * a.H * a.D8 + head * a.D8 + min(col, D - 1)]) : 0.0f;
    const unsigned lds0 = (unsigned)(size_t)(__attribute__((address_space(3))) void *)s_ring + (unsigned)(wave * L::WAVE);
    auto scalar = [&](const void *p) {
        const unsigned long long v = (unsigned long long)(uintptr_t)p;
        return (unsigned long long)(unsigned)__builtin_amdgcn_readfirstlane((int)(unsigned)v) | ((unsigned long long)(unsigned)__builtin_amdgcn_readfirstlane((int)(unsigned)(v >> 32)) << 32);
    };
    auto fetch = [&](int cc, int at) {  // chunk cc (behind the end: the last one again, the waits count instructions) into ring slot `at`
        const int c = min(cc, c_hi - 1);
        const unsigned dst0 = lds0 + (unsigned)(at * L::SLOT);
        const unsigned long long base = scalar(ws + (size_t)c * a.H * per);
        auto piece = [&](unsigned byte, unsigned dst) {
            unsigned keep;
            asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %3\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, %2\n\ts_mov_b32 m0, %0"
                         : "=&s"(keep)
                         : "v"(byte + (unsigned)lane * 16u), "s"(base), "s"(dst)
                         : "memory");
        };
#pragma unroll
        for (int j = 0; j < NB; ++j) {
            const int b = min(wave * NB + j, nblk - 1);  // (blocks past the end meet channels that stay zero)
#pragma unroll
            for (int k = 0; k < 4; ++k) piece((unsigned)(k * nblk + b) * 1024u, dst0 + (unsigned)(4 * j + k) * 1024u);
        }
        piece((unsigned)nblk * 4096u + (unsigned)min(wave, 2) * 1024u, dst0 + 4096u * NB);
        piece((unsigned)nblk * 4096u + 3072u, dst0 + 4096u * NB + 1024u);  // W_16 of all channels (and what lies behind it)
        const unsigned long long vbase = scalar(vp + (size_t)(DC * c) * a.ld * sizeof(T));
#pragma unroll
        for (int k = 0; k < L::VI; ++k) {
            const int t = min((64 / L::DW) * k + lane / L::DW, run.n_rows - 1 - DC * c);
            const unsigned off = (unsigned)(t * a.ld) * (unsigned)sizeof(T) + (unsigned)(lane % L::DW) * 4u;
            unsigned keep;
            asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %3\n\ts_nop 0\n\tglobal_load_lds_dword %1, %2\n\ts_mov_b32 m0, %0"
                         : "=&s"(keep)
                         : "v"(off), "s"(vbase), "s"(dst0 + 4096u * NB + 2048u + 256u * k)
                         : "memory");
        }
    };
    const dr_f32x4 zero = {0.0f, 0.0f, 0.0f, 0.0f};
    auto store_o = [&](int c) {  // chunk c's outputs: one per thread
        const float *p = (const float *)s_o[c % L::PB] + threadIdx.x;
        const float o = (p[0] + p[256]) + (p[512] + p[768]);
        const int l = threadIdx.x >> 2, t = DC * c + 4 * (l >> 4) + (threadIdx.x & 3), d = 16 * cb + (l & 15);
        if (t < run.n_rows && d < D) a.o[((size_t)(run.row0 + t) * a.H + head) * a.D8 + d] = o;
    };
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // (the state's loads: the waits below count DMAs)
#pragma unroll
    for (int i = 0; i < L::RING - 1; ++i) fetch(c_lo + i, i);
    int at = 0;
    for (int c = c_lo; c < c_hi; ++c) {
        asm volatile("s_waitcnt vmcnt(%0)" ::"n"((L::RING - 2) * L::OPS) : "memory");
        fetch(c + L::RING - 1, at ? at - 1 : L::RING - 1);  // into the previous chunk's slot
        const char *mine = s_ring + at * L::SLOT + wave * L::WAVE;
        at = at + 1 < L::RING ? at + 1 : 0;
        auto operand = [&](int piece) { return *(const dr_f32x4 *)(mine + piece * 1024 + lane * 16); };
        dr_f32x4 u[NB], r[NB], k[NB], m[NB], w[NB], v, x = operand(4 * NB);
#pragma unroll
        for (int j = 0; j < NB; ++j) u[j] = operand(4 * j);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = 4 * q + i;
            const float e = E::load((const T *)(mine + (4 * NB + 2) * 1024) + t * 16 + n16) + vbias;
            v[i] = DC * c + t < run.n_rows && col < D ? e : 0.0f;
        }
#pragma unroll
        for (int j = 0; j < NB; ++j) r[j] = operand(4 * j + 1), k[j] = operand(4 * j + 2), w[j] = *(const dr_f32x4 *)(mine + (4 * NB + 1) * 1024 + (16 * min(wave * NB + j, nblk - 1) + 4 * q) * 4);
        dr_f32x4 P = zero, O = zero;
#pragma unroll
        for (int j = 0; j < NB; ++j)
#pragma unroll
            for (int i = 0; i < 4; ++i) P = dr_mfma(u[j][i], S[j][i], P);
        if (wave == 0)
#pragma unroll
            for (int i = 0; i < 4; ++i) P = dr_mfma(x[i], v[i], P);
        s_p[c % L::PB][wave][lane] = P;
#pragma unroll
        for (int j = 0; j < NB; ++j) m[j] = operand(4 * j + 3);
#pragma unroll
        for (int j = 0; j < NB; ++j)
#pragma unroll
            for (int i = 0; i < 4; ++i) O = dr_mfma(r[j][i], S[j][i], O);
        if (wave == 1)
#pragma unroll
            for (int i = 0; i < 4; ++i) O = dr_mfma(x[i], v[i], O);
#pragma unroll
        for (int j = 0; j < NB; ++j) S[j] *= w[j];
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int j = 0; j < NB; ++j) S[j] = dr_mfma(k[j][i], v[i], S[j]);
        // the four waves' shares of P meet (LDS only: the DMAs stay in flight)
        asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
        P = (s_p[c % L::PB][0][lane] + s_p[c % L::PB][1][lane]) + (s_p[c % L::PB][2][lane] + s_p[c % L::PB][3][lane]);
        if (c > c_lo) store_o(c - 1);
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int j = 0; j < NB; ++j) S[j] = dr_mfma(m[j][i], P[i], S[j]);
        if (wave == 2)
#pragma unroll
            for (int i = 0; i < 4; ++i) O = dr_mfma(x[i], P[i], O);
#pragma unroll
        for (int j = 0; j < NB; ++j)
            if (wave * NB + j >= nblk) S[j] = zero;  // (a block that does not exist saw another's operands)
        if constexpr (L::PB == 1) asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");  // everyone has read P and the previous outputs
        s_o[c % L::PB][wave][lane] = O;
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // the look-ahead DMAs: LDS is handed on when the workgroup ends
    __syncthreads();
    store_o(c_hi - 1);
#pragma unroll
    for (int j = 0; j < NB; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int d = 16 * (wave * NB + j) + 4 * q + i;
            if (d < D && col < D) state[(size_t)d * D + col] = S[j][i];
        }
}

// chunks whose operands are made and used at a time
int delta_segment(int H, int D) {
    const size_t bytes = H * dr_chunk_floats(D) * 4;
    return (int)std::max((size_t)16, DELTA_SEGMENT_BYTES / bytes);
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
    DeltaArgs seg = a;
    const int step = delta_segment(a.H, a.D);
    for (int c = 0; c < chunks; c += step) {  // a segment's operands are read back before they leave the last-level cache
        seg.chunk_lo = c, seg.chunk_hi = std::min(chunks, c + step);
        hipLaunchKernelGGL((k_delta_prep<E, NB>), dim3((unsigned)a.H, (unsigned)(seg.chunk_hi - c)), dim3(256), lds, st, seg);
        PIE_LAUNCH_CHECK();
        hipLaunchKernelGGL((k_delta_scan<E, NB>), dim3((unsigned)(a.H * dr_blocks(a.D)), (unsigned)a.n_runs), dim3(256), 0, st, seg);
        PIE_LAUNCH_CHECK();
    }
    const int g0 = 3 * a.H * a.D8;
    const HeadOutArgs h = {a.o, nullptr, (const typename E::type *)a.raw + g0, a.bias ? a.bias + g0 : nullptr, a.ld, a.H, a.D, a.D8, a.o_norm, a.eps, a.out, a.ld_out};
    return head_out_launch(sizeof(typename E::type) == 4 ? PIE_F32 : PIE_BF16, h, row0, rows, st);
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
    const bool ahead = (long)a.n_runs * a.H <= 256 && a.D <= 128;
#define DS_GO(CP_, NT_) \
    if (ahead) hipLaunchKernelGGL((k_delta_step<E, CP_, NT_, CP_ <= 128>), grid, dim3(NT_), 0, st, a); \
    else hipLaunchKernelGGL((k_delta_step<E, CP_, NT_, false>), grid, dim3(NT_), 0, st, a)
    if (a.D <= 16) { DS_GO(16, 128); }
    else if (a.D <= 32) { DS_GO(32, 256); }
    else if (a.D <= 64) { DS_GO(64, 256); }
    else if (a.D <= 128) { DS_GO(128, 512); }
    else { DS_GO(256, 1024); }
#undef DS_GO
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

}  // namespace

int delta_chunks(int n_rows) { return (n_rows + DC - 1) / DC; }
size_t delta_ws_floats(int chunks, int H, int D) { return (size_t)std::min(chunks, delta_segment(H, D)) * H * dr_chunk_floats(D); }
int delta_launches(int chunks, int H, int D) { return 2 * ((chunks + delta_segment(H, D) - 1) / delta_segment(H, D)) + 1; }

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
