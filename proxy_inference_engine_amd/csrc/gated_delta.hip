// gated_delta.hip -- the gated delta rule (PIE_MIXER_GATED_DELTA): per head a state S [key channel][value column] in fp32, carried from token to token,
//   S <- g_t S,   u_t = b_t (v_t - S^T k_t),   S <- S + k_t u_t^T,   o_t = S^T q_t,
// with one decay g = exp(-rate softplus(. + bias)) and one step size b = sigmoid(.) per head and token, unit queries and keys shared by the heads of a group, and a short causal
// convolution with silu in front of q, k and v.
//
// The convolution's last inputs are kept as a ring, position p at p mod taps: a step reads taps - 1 places and writes the one that nobody reads, so the heads that share
// channels need no order between them.  Where every run is one row the step form convolves on the way; else one launch (k_gated_conv) does it for all rows.
//
// Step form (decoded tokens, short runs): one workgroup per (run, head), the state in registers, a thread RPT key channels of one value column; norm and gate in the same launch
// (heads of more than 256 columns: several workgroups, and head_out.hip behind them).
//
// Chunk form (longer runs), 16 tokens at a time.  With L_t the sum of the log decays inside the chunk up to t and S the state in front of it,
//   u_t = b_t v_t - b_t e^{L_t} S^T k_t - sum_{i<t} B_ti u_i,     B_ti = b_t e^{L_t - L_i} k_t . k_i
//   o_t = e^{L_t} S^T q_t + sum_{i<=t} e^{L_t - L_i} (q_t . k_i) u_i,     S <- e^{L_16} S + sum_i e^{L_16 - L_i} k_i u_i^T
// where no exponent is above zero, whatever the decays.  With T = (I + B)^-1 the u of a chunk are T b v - T b e^L K S: one launch (all chunks of all heads in parallel) leaves -T b e^L K, e^L Q, K,
// T b and the weighted Q K^T in matrix operand order, a second walks the chunks (chunk_scan.hpp, SCAN_GATED), a third takes the heads' norm and gate.
#include "chunk_scan.hpp"

namespace {

__device__ __forceinline__ float *gated_state(const GatedDeltaArgs &a, int m) {
    return a.state + min((unsigned)a.slots[min(a.row_seq[m], a.n_seqs - 1)], (unsigned)a.n_slots - 1u) * a.slot_floats;
}
struct GatedStep {
    float log_g, b;
};
template <class E>
__device__ __forceinline__ GatedStep gated_step(const GatedDeltaArgs &a, size_t m, int head) {
    typedef typename E::type T;
    constexpr bool F32 = sizeof(T) == 4;
    const T *p = (const T *)a.raw + m * a.ld + 2 * a.G * a.D8 + 2 * a.H * a.V8 + head;
    return {-a.decay_rate[head] * stack_softplus<F32>(E::load(p + a.H8) + a.decay_bias[head]), stack_sigmoid<F32>(E::load(p))};
}

// ---------------------------------------------------------------- the convolution over runs
template <class E>
__device__ __forceinline__ float4 gc_load(const typename E::type *p) {
    if constexpr (sizeof(typename E::type) == 4) return *(const float4 *)p;
    else {
        const uint2 v = *(const uint2 *)p;
        return make_float4(lo_f32<BF16>(v.x), hi_f32<BF16>(v.x), lo_f32<BF16>(v.y), hi_f32<BF16>(v.y));
    }
}

// TAPS: taps at most.  A thread owns four channels and walks the rows of a tile with the last inputs in registers; the run's first tile carries the ring.
template <class E, int TAPS>
__global__ void __launch_bounds__(256) k_gated_conv(const GatedDeltaArgs a, int C) {
    typedef typename E::type T;
    constexpr bool F32 = sizeof(T) == 4;
    const int n = (blockIdx.x * 256 + threadIdx.x) * 4, taps = a.taps;
    const RowChunk c = row_chunk(a.runs, a.n_runs, blockIdx.y, CONV_ROWS);
    if (c.n <= 0 || n >= C) return;
    const int run0 = c.row0 - c.pos, pos0 = a.pos[run0];
    float *ring = taps > 1 ? gated_state(a, run0) + a.ring + n : nullptr;
    const T *x = (const T *)a.raw + n;
    auto at = [&](int i) -> float4 {  // input i of the run; below zero: what the sequence had before
        if (i >= 0) return gc_load<E>(x + (size_t)(run0 + i) * a.ld);
        if (pos0 + i < 0 || i < 1 - taps) return make_float4(0, 0, 0, 0);
        return *(const float4 *)(ring + (size_t)((pos0 + i) % taps) * C);
    };
    float4 w[TAPS], v[TAPS];  // v[TAPS - 1]: the row itself
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
        const int i = j - (TAPS - taps);
        w[j] = i >= 0 ? *(const float4 *)(a.conv + (size_t)i * a.ldw + n) : make_float4(0, 0, 0, 0);
        v[j] = j > 0 ? at(c.pos + j - TAPS) : make_float4(0, 0, 0, 0);
    }
    if (c.pos == 0 && taps > 1) {  // (the old inputs have been read)
        const int n_rows = a.runs[c.run].n_rows;
        for (int i = max(0, n_rows - taps); i < n_rows; ++i) *(float4 *)(ring + (size_t)((pos0 + i) % taps) * C) = at(i);
    }
    constexpr int AHEAD = 8;  // rows in flight
    float4 r[AHEAD];
#pragma unroll
    for (int i = 0; i < CONV_ROWS; ++i) {
        if (i % AHEAD == 0)
#pragma unroll
            for (int k = 0; k < AHEAD; ++k) r[k] = gc_load<E>(x + (size_t)(c.row0 + min(i + k, c.n - 1)) * a.ld);
        if (i >= c.n) break;
#pragma unroll
        for (int j = 0; j + 1 < TAPS; ++j) v[j] = v[j + 1];
        v[TAPS - 1] = r[i % AHEAD];
        float4 y = make_float4(0, 0, 0, 0);
#pragma unroll
        for (int j = 0; j < TAPS; ++j) y = make_float4(fmaf(w[j].x, v[j].x, y.x), fmaf(w[j].y, v[j].y, y.y), fmaf(w[j].z, v[j].z, y.z), fmaf(w[j].w, v[j].w, y.w));
        y = make_float4(stack_silu<F32>(y.x), stack_silu<F32>(y.y), stack_silu<F32>(y.z), stack_silu<F32>(y.w));
        T *out = (T *)a.mixed + (size_t)(c.row0 + i) * C + n;
        if constexpr (F32) *(float4 *)out = y;
        else *(uint2 *)out = make_uint2(pack2<BF16>(y.x, y.y), pack2<BF16>(y.z, y.w));
    }
}

// ---------------------------------------------------------------- step form
// A token's inputs leave first, the state behind them: the convolution, the lengths and the exchanges of the first token run while the state is still on its way.
// CV: value columns of a workgroup; RPT: key channels per thread (RPT * NT / CV >= D)
template <class E, int CV, int NT, int RPT>
__global__ void __launch_bounds__(NT, 4) k_gated_step(const GatedDeltaArgs a) {
    typedef typename E::type T;
    constexpr bool F32 = sizeof(T) == 4;
    constexpr int SL = NT / CV, RP = RPT * SL, NI = (2 * RP + 2 * CV + NT - 1) / NT, AHEAD = 3;  // AHEAD: older inputs of the convolution that travel with the token's own
    static_assert(NT % CV == 0 && CV % 64 == 0 && RP % 64 == 0, "slices");
    __shared__ __attribute__((aligned(16))) float s_q[RP], s_k[RP], s_v[CV], s_g[CV], s_p[SL][CV], s_o[SL][CV], s_ss[CV / 64];
    const int head = blockIdx.y, D = a.D, V = a.V, lane = threadIdx.x & 63, w0 = __builtin_amdgcn_readfirstlane((int)threadIdx.x), group = head / (a.H / a.G), c0 = CV * blockIdx.z;
    const RowRun run = a.runs[blockIdx.x];
    const int c = threadIdx.x % CV, col = c0 + c, slice = w0 / CV, d0 = slice * RPT, C = gated_delta_channels(a.H, a.G, a.D8, a.V8), taps = a.taps;
    float *slot = gated_state(a, run.row0), *state = slot + (size_t)head * D * V, *ring = slot + a.ring;
    const int pos0 = a.pos[run.row0], at = pos0 % taps;
    const bool convolve = !a.mixed;

    // what the wave's lanes fetch: q, k, v, gate (what lies past a head: its last number, dropped afterwards)
    struct Place {
        int kind, i, ch;  // 0 .. 3, 4: nothing; index in LDS; column of raw
        bool live;
    };
    auto place = [&](int n) -> Place {
        const int first = w0 + n * NT, kind = first < RP ? 0 : first < 2 * RP ? 1 : first < 2 * RP + CV ? 2 : first < 2 * RP + 2 * CV ? 3 : 4;
        const int i = first + lane - (kind == 0 ? 0 : kind == 1 ? RP : kind == 2 ? 2 * RP : 2 * RP + CV), d = i + (kind >= 2 ? c0 : 0), size = kind >= 2 ? V : D;
        const int base = kind == 0 ? group * a.D8 : kind == 1 ? (a.G + group) * a.D8 : 2 * a.G * a.D8 + (kind == 3 ? a.H + head : head) * a.V8;
        return {kind, i, base + min(d, size - 1), d < size};
    };
    float now[NI], w[NI][AHEAD + 1], old[NI][AHEAD], raw_b, raw_a;
    auto fetch = [&](size_t m) {
        const T *x = (const T *)a.raw + m * a.ld;
#pragma unroll
        for (int n = 0; n < NI; ++n) {
            const Place p = place(n);
            if (p.kind == 4) continue;
            now[n] = E::load(p.kind == 3 || convolve ? x + p.ch : (const T *)a.mixed + m * C + p.ch);
            if (p.kind == 3 || !convolve) continue;
            w[n][AHEAD] = a.conv[(size_t)(taps - 1) * a.ldw + p.ch];
            if (taps > 1)
#pragma unroll
                for (int k = 0; k < AHEAD; ++k) {
                    const int back = min(k + 1, taps - 1);
                    w[n][k] = a.conv[(size_t)(taps - 1 - back) * a.ldw + p.ch], old[n][k] = ring[(size_t)(at < back ? at + taps - back : at - back) * C + p.ch];
                }
        }
        const T *p = x + C + a.H * a.V8 + head;
        raw_b = E::load(p), raw_a = E::load(p + a.H8);
    };
    auto place_inputs = [&] {
#pragma unroll
        for (int n = 0; n < NI; ++n) {
            const Place p = place(n);
            if (p.kind == 4) continue;
            float v = now[n];
            if (p.kind == 3) v = stack_silu<F32>(v);
            else if (convolve) {
                v *= w[n][AHEAD];
#pragma unroll
                for (int k = 0; k < AHEAD; ++k)
                    if (k + 1 < taps && pos0 > k) v = fmaf(w[n][k], old[n][k], v);
                for (int back = AHEAD + 1; back < taps; ++back)
                    if (pos0 >= back) v = fmaf(a.conv[(size_t)(taps - 1 - back) * a.ldw + p.ch], ring[(size_t)(at < back ? at + taps - back : at - back) * C + p.ch], v);
                if (taps > 1 && p.live && (p.kind == 2 || (head % (a.H / a.G) == 0 && blockIdx.z == 0))) ring[(size_t)at * C + p.ch] = now[n];
                v = stack_silu<F32>(v);
                if constexpr (!F32) v = round_T<BF16>(v);  // (as the launch that convolves runs leaves it)
            }
            (p.kind == 0 ? s_q : p.kind == 1 ? s_k : p.kind == 2 ? s_v : s_g)[p.i] = p.live ? v : 0.0f;
        }
    };
    fetch(run.row0);
    const float rate = a.decay_rate[head], bias = a.decay_bias[head], o_norm = a.o_norm[min(col, V - 1)];
    __builtin_amdgcn_sched_barrier(0);
    float S[RPT];
    const unsigned row4 = 4u * (unsigned)V;
    unsigned at0 = 4u * (unsigned)min(col, V - 1) + (unsigned)min(d0, D - 1) * row4;  // bytes: a head's state is at most 2 MiB
    {
        unsigned off = at0;
#pragma unroll
        for (int i = 0; i < RPT; ++i) S[i] = *(const float *)((const char *)state + off), off += d0 + i + 1 < D ? row4 : 0u;
    }  // (rows past D meet keys and queries of zero)
    __builtin_amdgcn_sched_barrier(0);

    for (int j = 0; j < run.n_rows; ++j) {
        const size_t m = run.row0 + j;
        place_inputs();
        const float g = stack_exp<F32>(-rate * stack_softplus<F32>(raw_a + bias)), b = stack_sigmoid<F32>(raw_b);
        lds_barrier();
        float qq = 0.0f, kk = 0.0f;  // every wave: the lengths
        for (int d = lane; d < RP; d += 64) qq = fmaf(s_q[d], s_q[d], qq), kk = fmaf(s_k[d], s_k[d], kk);
        const float uq = a.scale / sqrtf(lanes_sum(qq) + a.unit_eps), uk = 1.0f / sqrtf(lanes_sum(kk) + a.unit_eps);
        if (j == 0 && pos0 == 0)
#pragma unroll
            for (int i = 0; i < RPT; ++i) S[i] = 0.0f;
        float p = 0.0f;
#pragma unroll
        for (int i = 0; i < RPT; ++i) {
            p = fmaf(s_k[d0 + i], S[i], p);
            if (i % 8 == 7) __builtin_amdgcn_sched_barrier(0);  // (else all the vectors' numbers are in registers at once)
        }
        s_p[slice][c] = p;
        lds_barrier();
        p = 0.0f;
#pragma unroll
        for (int i = 0; i < SL; ++i) p += s_p[i][c];
        const float u = b * (s_v[c] - g * (p * uk)) * uk;
        float o = 0.0f;
#pragma unroll
        for (int i = 0; i < RPT; ++i) {
            S[i] = fmaf(s_k[d0 + i], u, g * S[i]);
            o = fmaf(s_q[d0 + i], S[i], o);
            if (i % 8 == 7) __builtin_amdgcn_sched_barrier(0);
        }
        s_o[slice][c] = o * uq;
        if (j + 1 < run.n_rows) fetch(m + 1);
        else if (col < V)  // the state leaves while the output is finished
        {
            asm volatile("" : "+v"(at0));  // (the addresses are made again: kept since the loads, they would take a register each)
#pragma unroll
            for (int i = 0; i < RPT; ++i, at0 += row4)
                if (d0 + i < D) *(float *)((char *)state + at0) = S[i];
        }
        lds_barrier();
        if (gridDim.z > 1) {  // norm and gate need the other workgroups' columns too
            if (threadIdx.x < CV && col < V) {
                o = 0.0f;
#pragma unroll
                for (int i = 0; i < SL; ++i) o += s_o[i][c];
                a.o[(m * a.H + head) * a.V8 + col] = o;
            }
            continue;  // (s_o is written again behind the next token's barriers)
        }
        if (threadIdx.x < CV) {  // whole waves
            o = 0.0f;
#pragma unroll
            for (int i = 0; i < SL; ++i) o += s_o[i][c];
            o = col < V ? o : 0.0f;
            const float sum = lanes_sum(o * o);
            if (lane == 0) s_ss[threadIdx.x >> 6] = sum;
        }
        lds_barrier();
        if (threadIdx.x < CV && col < V) {
            float sum = s_ss[0];
#pragma unroll
            for (int i = 1; i < CV / 64; ++i) sum += s_ss[i];
            ((T *)a.out)[m * a.ld_out + head * a.V8 + col] = E::pack(o * (1.0f / sqrtf(sum / (float)V + a.eps)) * o_norm * s_g[c]);
        }
        lds_barrier();  // the vectors are written again
    }
}

// ---------------------------------------------------------------- chunk form: the operands
// One workgroup per (chunk, head).  A wave owns four tokens; its lanes own channel pairs.  NB: 16-channel blocks per wave in the products (D <= 64 NB).
template <class E, int NB>
__global__ void __launch_bounds__(256) k_gated_prep(const GatedDeltaArgs a, int chunk_lo) {
    typedef typename E::type T;
    constexpr bool F32 = sizeof(T) == 4;
    constexpr int LD = 64 * NB + 4, NP = (NB + 1) / 2, TP = DC / 4, LM = 20;
    __shared__ __attribute__((aligned(16))) float s_q[DC * LD], s_k[DC * LD], s_b[DC * LM], s_y[DC * LM], s_t[DC * LM], s_l[DC], s_step[DC];
    const int D = a.D, nblk = dr_blocks(D), lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), n16 = lane & 15, q = lane >> 4;
    const int head = blockIdx.x, group = head / (a.H / a.G), C = gated_delta_channels(a.H, a.G, a.D8, a.V8);
    const ScanChunk c = scan_chunk(a.runs, a.n_runs, chunk_lo + (int)blockIdx.y);
    if (c.n <= 0) return;
    ElemPair xq[NP][TP], xk[NP][TP];
#pragma unroll
    for (int p = 0; p < NP; ++p) {
        const int d = min(2 * (lane + 64 * p), a.D8 - 2);
#pragma unroll
        for (int j = 0; j < TP; ++j) {
            const T *x = (const T *)a.mixed + (size_t)(c.row0 + min(TP * wave + j, c.n - 1)) * C + group * a.D8 + d;
            xq[p][j] = load_pair<E>(x), xk[p][j] = load_pair<E>(x + a.G * a.D8);
        }
    }
    if (wave == 0) {  // lane t: the running sum of the log decays (rows past the end: no decay, no step)
        GatedStep st = gated_step<E>(a, c.row0 + min(n16, c.n - 1), head);
        if (n16 >= c.n) st = {0.0f, 0.0f};
        float l = st.log_g;
#pragma unroll
        for (int o = 1; o < DC; o <<= 1) {
            const float v = __shfl_up(l, o, DC);
            if (n16 >= o) l += v;
        }
        if (lane < DC) s_l[lane] = l, s_step[lane] = st.b;
    }
#pragma unroll
    for (int j = 0; j < TP; ++j) {
        const int t = TP * wave + j;
        float qq = 0.0f, kk = 0.0f;
#pragma unroll
        for (int p = 0; p < NP; ++p) {
            const int d = 2 * (lane + 64 * p);
            if (d >= D || t >= c.n) xq[p][j].x = xk[p][j].x = 0.0f;
            if (d + 1 >= D || t >= c.n) xq[p][j].y = xk[p][j].y = 0.0f;
            qq = fmaf(xq[p][j].x, xq[p][j].x, fmaf(xq[p][j].y, xq[p][j].y, qq)), kk = fmaf(xk[p][j].x, xk[p][j].x, fmaf(xk[p][j].y, xk[p][j].y, kk));
        }
        const float uq = a.scale / sqrtf(lanes_sum(qq) + a.unit_eps), uk = 1.0f / sqrtf(lanes_sum(kk) + a.unit_eps);
#pragma unroll
        for (int p = 0; p < NP; ++p) {
            const int d = 2 * (lane + 64 * p);
            if (d >= 16 * nblk) break;
            *(float2 *)(s_q + t * LD + d) = make_float2(xq[p][j].x * uq, xq[p][j].y * uq);
            *(float2 *)(s_k + t * LD + d) = make_float2(xk[p][j].x * uk, xk[p][j].y * uk);
        }
    }
    lds_barrier();
    if (wave < 2) {  // wave 0: B (transposed), 1: the weighted Q K^T
        const float *l = wave == 0 ? s_k : s_q;
        dr_f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
        for (int b = 0; b < nblk; ++b) {
            const dr_f32x4 lv = *(const dr_f32x4 *)(l + n16 * LD + 16 * b + 4 * q), rv = *(const dr_f32x4 *)(s_k + n16 * LD + 16 * b + 4 * q);
#pragma unroll
            for (int i = 0; i < 4; ++i) acc = dr_mfma(lv[i], rv[i], acc);
        }
        const float li = s_l[n16];
#pragma unroll
        for (int i = 0; i < 4; ++i) {  // row t, column n16
            const int t = 4 * q + i;
            const float w = n16 < t + wave ? stack_exp<F32>(s_l[t] - li) * (wave == 0 ? s_step[t] : 1.0f) : 0.0f;
            acc[i] = n16 < t + wave ? acc[i] * w : 0.0f;
        }
        if (wave == 0) *(dr_f32x4 *)(s_b + n16 * LM + 4 * q) = acc;
        else
#pragma unroll
            for (int i = 0; i < 4; ++i) s_y[(4 * q + i) * LM + n16] = acc[i];
    }
    lds_barrier();
    float *out = a.ws + ((size_t)blockIdx.y * a.H + head) * scan_chunk_floats(SCAN_GATED, D);
    float *o_r = out + nblk * 256, *o_k = o_r + nblk * 256, *o_m = o_k + nblk * 256;
    const float l_end = s_l[DC - 1];
    if (wave == 0) {
        float tc[DC];
        scan_inverse<LM>(s_b, n16, tc);
        if (q == 0)
#pragma unroll
            for (int t = 0; t < DC; ++t) s_t[t * LM + n16] = tc[t] * s_step[n16];  // T b
        *(dr_f32x4 *)(o_m + lane * 4) = *(const dr_f32x4 *)(s_t + n16 * LM + 4 * q);
    } else {
        const float e = stack_exp<F32>(s_l[n16]);
        float back[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) back[i] = stack_exp<F32>(l_end - s_l[4 * q + i]);
        for (int b = wave - 1; b < nblk; b += 3) {
            *(dr_f32x4 *)(o_r + b * 256 + lane * 4) = *(const dr_f32x4 *)(s_q + n16 * LD + 16 * b + 4 * q) * e;
            dr_f32x4 k;
#pragma unroll
            for (int i = 0; i < 4; ++i) k[i] = s_k[(4 * q + i) * LD + 16 * b + n16] * back[i];
            *(dr_f32x4 *)(o_k + b * 256 + lane * 4) = k;
        }
        if (wave == 2) *(dr_f32x4 *)(o_m + 256 + lane * 4) = *(const dr_f32x4 *)(s_y + n16 * LM + 4 * q);
        if (wave == 3) {
            const float w = stack_exp<F32>(l_end);
            for (int d = lane; d < 16 * nblk; d += 64) o_m[512 + d] = w;
        }
    }
    lds_barrier();
    dr_f32x4 tv = *(const dr_f32x4 *)(s_t + n16 * LM + 4 * q);
#pragma unroll
    for (int i = 0; i < 4; ++i) tv[i] *= -stack_exp<F32>(s_l[4 * q + i]);
#pragma unroll
    for (int j = 0; j < NB; ++j) {
        const int b = wave * NB + j;
        if (b >= nblk) break;
        dr_f32x4 u = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int i = 0; i < 4; ++i) u = dr_mfma(s_k[(4 * q + i) * LD + 16 * b + n16], tv[i], u);  // (-T b e^L K)^T
        *(dr_f32x4 *)(out + b * 256 + lane * 4) = u;
    }
}

HeadOutArgs gated_head_out(const GatedDeltaArgs &a, size_t elem) {
    return {a.o, nullptr, (const char *)a.raw + (size_t)gated_delta_channels(a.H, a.G, a.D8, a.V8) * elem, nullptr, a.ld, a.H, a.V, a.V8, a.o_norm, a.eps, a.out, a.ld_out, true, true, 1.0f};
}

template <class E, int NB>
int gated_chunks_nb(const GatedDeltaArgs &a, int chunks, hipStream_t st) {
    typedef typename E::type T;
    const int C = gated_delta_channels(a.H, a.G, a.D8, a.V8);
    const ScanArgs scan = {(const T *)a.mixed + 2 * a.G * a.D8, nullptr, C, a.H, a.D, a.V, a.V8, a.pos, a.row_seq, a.slots, a.n_seqs, a.n_slots, a.runs, a.n_runs, a.state, a.slot_floats, a.ws, a.o, 0, 0};
    return scan_chunks<E, NB, SCAN_GATED>(scan, chunks, st, [&](int lo, int hi) {
        hipLaunchKernelGGL((k_gated_prep<E, NB>), dim3((unsigned)a.H, (unsigned)(hi - lo)), dim3(256), 0, st, a, lo);
    });
}
template <class E>
int gated_chunks_go(const GatedDeltaArgs &a, int chunks, hipStream_t st) {
    if (a.D <= 64) return gated_chunks_nb<E, 1>(a, chunks, st);
    if (a.D <= 128) return gated_chunks_nb<E, 2>(a, chunks, st);
    if (a.D <= 192) return gated_chunks_nb<E, 3>(a, chunks, st);
    return gated_chunks_nb<E, 4>(a, chunks, st);
}

template <class E>
int gated_step_go(const GatedDeltaArgs &a, hipStream_t st) {
    const int cv = a.V <= 64 ? 64 : a.V <= 128 ? 128 : 256;
    const dim3 grid((unsigned)a.n_runs, (unsigned)a.H, (unsigned)((a.V + cv - 1) / cv));
#define GS_GO(CV_, NT_, R_) hipLaunchKernelGGL((k_gated_step<E, CV_, NT_, R_>), grid, dim3(NT_), 0, st, a)
#define GS_D(CV_, NT_) \
    if (a.D <= 64) { GS_GO(CV_, NT_, 64 * CV_ / NT_); } \
    else if (a.D <= 128) { GS_GO(CV_, NT_, 128 * CV_ / NT_); } \
    else { GS_GO(CV_, NT_, 256 * CV_ / NT_); }
    if (cv == 64) { GS_D(64, 512); }
    else if (cv == 128 && a.D <= 128 && (long)a.n_runs * a.H > 256) { GS_D(128, 512); }
    else if (cv == 128) { GS_D(128, 1024); }
    else { GS_D(256, 1024); }
#undef GS_D
#undef GS_GO
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

template <class E>
void gated_conv_go(const GatedDeltaArgs &a, int tiles, hipStream_t st) {
    const int C = gated_delta_channels(a.H, a.G, a.D8, a.V8);
    const dim3 grid((unsigned)((C + 1023) / 1024), (unsigned)tiles);
#define GC_GO(T_) hipLaunchKernelGGL((k_gated_conv<E, T_>), grid, dim3(256), 0, st, a, C)
    if (a.taps <= 2) GC_GO(2);
    else if (a.taps == 3) GC_GO(3);
    else if (a.taps == 4) GC_GO(4);
    else if (a.taps <= 8) GC_GO(8);
    else GC_GO(16);
#undef GC_GO
}

int gated_check(const GatedDeltaArgs &a) {
    PIE_REQUIRE(a.D > 0 && a.D <= GATED_MAX_DIM && a.V > 0 && a.V <= HEAD_OUT_MAX_DIM && a.G > 0 && a.H % a.G == 0 && a.H <= 65535, PIE_E_SHAPE,
                "gated delta rule: keys of at most 256 numbers, values of at most 2048, a whole number of heads per key head");
    PIE_REQUIRE(a.taps > 0 && a.taps <= CONV_MAX_TAPS && a.conv && a.slots && a.state && a.n_slots > 0, PIE_E_ARG, "gated delta rule: a convolution of 1 .. 16 taps, and state slots");
    PIE_REQUIRE(a.ld % 8 == 0 && a.ldw % 4 == 0 && a.ring % 4 == 0 && a.slot_floats % 4 == 0, PIE_E_ALIGN, "gated delta rule: row strides");
    return PIE_OK;
}

}  // namespace

size_t gated_delta_ws_floats(int chunks, int H, int D) { return scan_ws_floats(SCAN_GATED, chunks, H, D); }
int gated_delta_chunk_launches(int chunks, int H, int D) { return scan_launches(SCAN_GATED, chunks, H, D) + 1; }

int gated_delta_conv_launch(int dtype, const GatedDeltaArgs &a, int tiles, hipStream_t st) {
    if (tiles <= 0) return PIE_OK;
    if (const int rc = gated_check(a)) return rc;
    PIE_REQUIRE(a.mixed && tiles <= 65535, PIE_E_ARG, "gated delta rule: the convolution of runs needs its buffer");
    if (dtype == PIE_F32) gated_conv_go<ElemF32>(a, tiles, st);
    else gated_conv_go<ElemBF16>(a, tiles, st);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

int gated_delta_step_launch(int dtype, const GatedDeltaArgs &a, int row0, int rows, hipStream_t st) {
    if (a.n_runs <= 0) return PIE_OK;
    if (const int rc = gated_check(a)) return rc;
    PIE_REQUIRE((a.mixed || a.n_runs == rows) && (a.V <= 256 || a.o), PIE_E_ARG, "gated delta rule: runs of several rows are convolved beforehand");
    if (const int rc = dtype == PIE_F32 ? gated_step_go<ElemF32>(a, st) : gated_step_go<ElemBF16>(a, st)) return rc;
    return a.V > 256 ? head_out_launch(dtype, gated_head_out(a, dtype == PIE_F32 ? 4 : 2), row0, rows, st) : PIE_OK;
}

int gated_delta_chunks_launch(int dtype, const GatedDeltaArgs &a, int chunks, int row0, int rows, hipStream_t st) {
    if (a.n_runs <= 0) return PIE_OK;
    if (const int rc = gated_check(a)) return rc;
    PIE_REQUIRE(a.mixed && a.ws && a.o && chunks > 0 && a.n_runs <= 65535, PIE_E_ARG, "gated delta rule: the chunk form needs its workspace");
    if (const int rc = dtype == PIE_F32 ? gated_chunks_go<ElemF32>(a, chunks, st) : gated_chunks_go<ElemBF16>(a, chunks, st)) return rc;
    return head_out_launch(dtype, gated_head_out(a, dtype == PIE_F32 ? 4 : 2), row0, rows, st);
}
