// time_mix.hip -- RWKV-6's time mixing (pie_stack_time_mix): per head a state S [key channel][value column] in fp32, carried from token to token,
//   o_t = (S_(t-1) + diag(u) k_t v_t^T)^T r_t,   S_t = diag(w_t) S_(t-1) + k_t v_t^T,
// with the decay w = exp(-exp(w2 tanh(.) + b)) per head and key channel, and a bonus u for the current token.  What it reads are projections of the token mixed with its
// predecessor (row_update.hip); every head's output over its root mean square, times a weight and the silu of its gate, goes to the output projection.
//
// Step form (decoded tokens, short runs): one workgroup per (run, head), the state in registers, a thread RPT key channels of one value column; decay, norm and gate on the way
// (heads of more than 128 channels: two workgroups, and head_out.hip behind them).
//
// Chunk form (longer runs), 16 tokens at a time.  With L_t the sum of the log decays inside the chunk up to t (per channel) and S the state in front of it,
//   o_t = S^T (e^{L_(t-1)} r_t) + sum_{i<=t} Y_ti v_i,   Y_ti = sum_d r_td k_id e^{L_(t-1) - L_i} for i < t,  sum_d r_td k_td u_d for i = t
//   S <- e^{L_16} S + sum_i (e^{L_16 - L_i} k_i) v_i^T
// One launch (all chunks of all heads in parallel) leaves e^L R, e^(L_16 - L) K and Y in matrix operand order, a second walks the chunks (chunk_scan.hpp, SCAN_LINEAR), a third
// takes norm and gate.  Decays may be as small as they like, so no quotient of products of decays is formed: between blocks of four tokens both factors of e^{L_(t-1) - L_i} are taken
// relative to the later block's start (no exponent above zero), inside a block the weights are products of at most two decays.
#include "chunk_scan.hpp"
#include "low_rank.hpp"

namespace {

__device__ __forceinline__ float *time_mix_state(const TimeMixArgs &a, const RowRun &run, int head) {
    return a.state + min((unsigned)a.slots[min(a.row_seq[run.row0], a.n_seqs - 1)], (unsigned)a.n_slots - 1u) * a.slot_floats + (size_t)head * a.D * a.D;
}

// ---------------------------------------------------------------- step form
// A token's inputs leave first, the state behind them: the decay and the exchanges of the first token run while the state is still on its way.
// CV: value columns of a workgroup; RPT: key channels per thread (RPT * NT / CV >= D)
template <class E, int CV, int NT, int RPT>
__global__ void __launch_bounds__(NT, 4) k_time_mix_step(const TimeMixArgs a) {
    typedef typename E::type T;
    constexpr bool F32 = sizeof(T) == 4;
    constexpr int SL = NT / CV, RP = RPT * SL, NI = (2 * RP + 2 * CV + NT - 1) / NT, CPT = (RP + NT / 8 - 1) / (NT / 8), WS = 2;  // WS: pieces of the decay's weights that travel with the token
    static_assert(NT % CV == 0 && CV % 64 == 0 && RP % 64 == 0, "slices");
    __shared__ __attribute__((aligned(16))) float s_r[RP], s_k[RP], s_w[RP], s_u[RP], s_v[CV], s_g[CV], s_low[TIME_MIX_MAX_RANK], s_o[SL][CV], s_ss[CV / 64];
    const int head = blockIdx.y, D = a.D, lane = threadIdx.x & 63, w0 = __builtin_amdgcn_readfirstlane((int)threadIdx.x), c0 = CV * blockIdx.z;
    const RowRun run = a.runs[blockIdx.x];
    const int c = threadIdx.x % CV, col = c0 + c, slice = w0 / CV, d0 = slice * RPT;
    float *state = time_mix_state(a, run, head);
    const bool fresh = a.pos[run.row0] == 0;

    // what the wave's lanes fetch: r, k, v, gate (what lies past a head: its last number, dropped afterwards)
    struct Place {
        int kind, i, d;  // 0 .. 3, 4: nothing; index in LDS; channel
        bool live;
    };
    auto place = [&](int n) -> Place {
        const int first = w0 + n * NT, kind = first < RP ? 0 : first < 2 * RP ? 1 : first < 2 * RP + CV ? 2 : first < 2 * RP + 2 * CV ? 3 : 4;
        const int i = first + lane - (kind == 0 ? 0 : kind == 1 ? RP : kind == 2 ? 2 * RP : 2 * RP + CV), d = i + (kind >= 2 ? c0 : 0);
        return {kind, i, min(d, D - 1), d < D};
    };
    float now[NI], low;
    auto fetch = [&](size_t m) {
#pragma unroll
        for (int n = 0; n < NI; ++n) {
            const Place p = place(n);
            if (p.kind < 4) now[n] = E::load((const T *)(p.kind == 0 ? a.r : p.kind == 1 ? a.k : p.kind == 2 ? a.v : a.gate) + m * a.ld + head * a.D8 + p.d);
        }
        low = E::load((const T *)a.low + m * a.ld_low + min((int)threadIdx.x, a.R8 - 1));
    };
    fetch(run.row0);
    uint4 wd[CPT][WS];  // eight lanes per channel
    float db[CPT];
    auto weights = [&](int d, int i) { return *(const uint4 *)(a.w_decay + (size_t)(head * D + min(d, D - 1)) * a.R8 + min(i, a.R8 - 8)); };
#pragma unroll
    for (int k = 0; k < CPT; ++k) {
        const int d = (threadIdx.x >> 3) + k * (NT / 8);
#pragma unroll
        for (int s = 0; s < WS; ++s) wd[k][s] = weights(d, (threadIdx.x & 7) * 8 + 64 * s);
        db[k] = a.decay_bias[head * D + min(d, D - 1)];
    }
    const float o_norm = a.o_norm[head * D + min(col, D - 1)];
    if (threadIdx.x < RP) s_u[threadIdx.x] = (int)threadIdx.x < D ? a.bonus[head * D + threadIdx.x] : 0.0f;
    __builtin_amdgcn_sched_barrier(0);
    float S[RPT];
    const unsigned row4 = 4u * (unsigned)D;
    unsigned at0 = 4u * (unsigned)min(col, D - 1) + (unsigned)min(d0, D - 1) * row4;  // bytes: a head's state is at most 2 MiB
    {
        unsigned off = at0;
#pragma unroll
        for (int i = 0; i < RPT; ++i) S[i] = *(const float *)((const char *)state + off), off += d0 + i + 1 < D ? row4 : 0u;
    }  // (rows past D meet r and k of zero)
    __builtin_amdgcn_sched_barrier(0);

    for (int j = 0; j < run.n_rows; ++j) {
        const size_t m = run.row0 + j;
#pragma unroll
        for (int n = 0; n < NI; ++n) {
            const Place p = place(n);
            if (p.kind < 4) (p.kind == 0 ? s_r : p.kind == 1 ? s_k : p.kind == 2 ? s_v : s_g)[p.i] = !p.live ? 0.0f : p.kind == 3 ? stack_silu<F32>(now[n]) : now[n];
        }
        if ((int)threadIdx.x < a.R8) s_low[threadIdx.x] = (int)threadIdx.x < a.rank ? stack_tanh<F32>(low) : 0.0f;
#pragma unroll 1
        for (int i = threadIdx.x + NT; i < a.R8; i += NT) s_low[i] = i < a.rank ? stack_tanh<F32>(E::load((const T *)a.low + m * a.ld_low + i)) : 0.0f;
        lds_barrier();
        auto part = [&](float z, int i, const uint4 &w) {
            const float4 l0 = *(const float4 *)(s_low + i), l1 = *(const float4 *)(s_low + i + 4);
            z = fmaf(lo_f32<BF16>(w.x), l0.x, fmaf(hi_f32<BF16>(w.x), l0.y, fmaf(lo_f32<BF16>(w.y), l0.z, fmaf(hi_f32<BF16>(w.y), l0.w, z))));
            return fmaf(lo_f32<BF16>(w.z), l1.x, fmaf(hi_f32<BF16>(w.z), l1.y, fmaf(lo_f32<BF16>(w.w), l1.z, fmaf(hi_f32<BF16>(w.w), l1.w, z))));
        };
#pragma unroll
        for (int k = 0; k < CPT; ++k) {
            const int d = (threadIdx.x >> 3) + k * (NT / 8);
            float z = 0.0f;
#pragma unroll
            for (int s = 0; s < WS; ++s)
                if ((int)(threadIdx.x & 7) * 8 + 64 * s < a.R8) z = part(z, (threadIdx.x & 7) * 8 + 64 * s, wd[k][s]);
#pragma unroll 1
            for (int i = (threadIdx.x & 7) * 8 + 64 * WS; i < a.R8; i += 64) z = part(z, i, weights(d, i));
            z = lanes8_sum(z);
            if ((threadIdx.x & 7) == 0 && d < RP) s_w[d] = d < D ? stack_exp<F32>(-stack_exp<F32>(z + db[k])) : 1.0f;
        }
        if (j == 0 && fresh)
#pragma unroll
            for (int i = 0; i < RPT; ++i) S[i] = 0.0f;
        const float v = s_v[c];
        float o = 0.0f;
#pragma unroll
        for (int i = 0; i < RPT; ++i) {
            o = fmaf(s_r[d0 + i], S[i], o);
            if (i % 8 == 7) __builtin_amdgcn_sched_barrier(0);  // (else all the vectors' numbers are in registers at once)
        }
        s_o[slice][c] = o;
        float bonus = 0.0f;  // of the current token: the waves that finish the outputs
        if (threadIdx.x < CV) {
            for (int d = lane; d < RP; d += 64) bonus = fmaf(s_r[d] * s_u[d], s_k[d], bonus);
            bonus = lanes_sum(bonus);
        }
        lds_barrier();
#pragma unroll
        for (int i = 0; i < RPT; ++i) {
            S[i] = fmaf(s_k[d0 + i], v, s_w[d0 + i] * S[i]);
            if (i % 8 == 7) __builtin_amdgcn_sched_barrier(0);
        }
        if (j + 1 < run.n_rows) fetch(m + 1);
        else if (col < D)  // the state leaves while the output is finished
        {
            asm volatile("" : "+v"(at0));  // (the addresses are made again: kept since the loads, they would take a register each)
#pragma unroll
            for (int i = 0; i < RPT; ++i, at0 += row4)
                if (d0 + i < D) *(float *)((char *)state + at0) = S[i];
        }
        if (threadIdx.x < CV) {  // whole waves
            o = bonus * v;
#pragma unroll
            for (int i = 0; i < SL; ++i) o += s_o[i][c];
            o = col < D ? o : 0.0f;
            if (gridDim.z > 1) {  // norm and gate need the other workgroups' columns too
                if (col < D) a.o[(m * a.H + head) * a.D8 + col] = o;
            } else {
                const float sum = lanes_sum(o * o);
                if (lane == 0) s_ss[threadIdx.x >> 6] = sum;
            }
        }
        lds_barrier();
        if (gridDim.z > 1) continue;
        if (threadIdx.x < CV && col < D) {
            float sum = s_ss[0];
#pragma unroll
            for (int i = 1; i < CV / 64; ++i) sum += s_ss[i];
            ((T *)a.out)[m * a.ld_out + head * a.D8 + col] = E::pack(o * (1.0f / sqrtf(sum / (float)D + a.eps)) * o_norm * s_g[c] * a.out_scale);
        }
        lds_barrier();  // the channel vectors are written again
    }
}

// ---------------------------------------------------------------- chunk form: the operands
// One workgroup per (chunk, head).  A wave owns four tokens; its lanes own channel pairs.  Dynamic LDS: see time_mix_prep_lds().
template <class E, int NB>
__global__ void __launch_bounds__(256) k_time_mix_prep(const TimeMixArgs a, int chunk_lo) {
    typedef typename E::type T;
    constexpr bool F32 = sizeof(T) == 4;
    constexpr int LD = 64 * NB + 4, NP = (NB + 1) / 2, TP = DC / 4, LM = 20;
    extern __shared__ __attribute__((aligned(16))) char lds[];
    float *s_l = (float *)lds, *s_y = s_l + DC * LD, *s_r = s_y + DC * LM, *s_k = s_r + DC * LD;  // log decays (then their running sums); Y; r, k
    // (the low-rank input of the decay lies where r and k come later)
    const int D = a.D, nblk = dr_blocks(D), lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), n16 = lane & 15, q = lane >> 4;
    const int head = blockIdx.x;
    const ScanChunk c = scan_chunk(a.runs, a.n_runs, chunk_lo + (int)blockIdx.y);
    if (c.n <= 0) return;
    const LowRankArgs low = {(const T *)a.low + (size_t)c.row0 * a.ld_low, a.ld_low, c.n, a.rank, a.R8, nullptr, a.w_decay + (size_t)head * D * a.R8, a.decay_bias + head * D, D};
    LowRank<E, NB> lr;
    lr.load(low);
    ElemPair xr[NP][TP], xk[NP][TP], u[NP];
#pragma unroll
    for (int p = 0; p < NP; ++p) {
        const int d = min(2 * (lane + 64 * p), a.D8 - 2);
#pragma unroll
        for (int j = 0; j < TP; ++j) {
            const size_t at = (size_t)(c.row0 + min(TP * wave + j, c.n - 1)) * a.ld + head * a.D8 + d;
            xr[p][j] = load_pair<E>((const T *)a.r + at), xk[p][j] = load_pair<E>((const T *)a.k + at);
        }
        u[p] = {a.bonus[head * D + min(d, D - 1)], a.bonus[head * D + min(d + 1, D - 1)]};
    }
    lr.load_weights(low, wave, lane);
    lr.put(low, s_r);
    lds_barrier();
    lr.product(low, s_r, wave, lane, [&](int t, int d, float z) { s_l[t * LD + d] = t < c.n && d < D ? -stack_exp<F32>(z) : 0.0f; });
    lds_barrier();  // the low-rank input has been read
    // the wave's own tokens: r and k into LDS, and the weights among themselves
    float y[TP][TP] = {};
#pragma unroll
    for (int p = 0; p < NP; ++p) {
        const int d = 2 * (lane + 64 * p);
        if (d >= 16 * nblk) break;
        float2 w[TP];  // (of the first and last token: not used)
#pragma unroll
        for (int j = 0; j < TP; ++j) {
            const int t = TP * wave + j;
            if (d >= D || t >= c.n) xr[p][j].x = xk[p][j].x = 0.0f;
            if (d + 1 >= D || t >= c.n) xr[p][j].y = xk[p][j].y = 0.0f;
            *(float2 *)(s_r + t * LD + d) = make_float2(xr[p][j].x, xr[p][j].y), *(float2 *)(s_k + t * LD + d) = make_float2(xk[p][j].x, xk[p][j].y);
            const float2 l = *(const float2 *)(s_l + t * LD + d);
            w[j] = make_float2(stack_exp<F32>(l.x), stack_exp<F32>(l.y));
        }
#pragma unroll
        for (int t = 0; t < TP; ++t) {
            y[t][t] = fmaf(xr[p][t].x * u[p].x, xk[p][t].x, fmaf(xr[p][t].y * u[p].y, xk[p][t].y, y[t][t]));
            float2 r = make_float2(xr[p][t].x, xr[p][t].y);  // times the decays between
#pragma unroll
            for (int i = t - 1; i >= 0; --i) {
                y[t][i] = fmaf(r.x, xk[p][i].x, fmaf(r.y, xk[p][i].y, y[t][i]));
                r.x *= w[i].x, r.y *= w[i].y;
            }
        }
    }
#pragma unroll
    for (int t = 0; t < TP; ++t)
#pragma unroll
        for (int i = 0; i < TP; ++i) {
            const float v = i <= t ? lanes_sum(y[t][i]) : 0.0f;
            if (lane == 0) s_y[(TP * wave + t) * LM + TP * wave + i] = v;
        }
    lds_barrier();
    for (int d = threadIdx.x; d < 16 * nblk; d += 256) {  // running sums
        float L = 0.0f;
#pragma unroll
        for (int t = 0; t < DC; ++t) L += s_l[t * LD + d], s_l[t * LD + d] = L;
    }
    lds_barrier();
    {  // the weights of the wave's tokens with those of the blocks in front of it
        dr_f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
        if (wave > 0)
            for (int b = 0; b < nblk; ++b) {
                const int d = 16 * b + 4 * q;
                const dr_f32x4 ref = *(const dr_f32x4 *)(s_l + (TP * wave - 1) * LD + d);
                dr_f32x4 rv = *(const dr_f32x4 *)(s_r + n16 * LD + d), kv = *(const dr_f32x4 *)(s_k + n16 * LD + d);
                const dr_f32x4 lr1 = *(const dr_f32x4 *)(s_l + max(n16 - 1, 0) * LD + d), lk = *(const dr_f32x4 *)(s_l + n16 * LD + d);
                const bool mine = n16 / TP == wave, before = n16 < TP * wave;
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    rv[i] = mine ? rv[i] * stack_exp<F32>(lr1[i] - ref[i]) : 0.0f, kv[i] = before ? kv[i] * stack_exp<F32>(ref[i] - lk[i]) : 0.0f;
                    acc = dr_mfma(rv[i], kv[i], acc);
                }
            }
        // row 4 q + i, column n16: the wave's rows are those of its quarter
        if (q == wave)
#pragma unroll
            for (int i = 0; i < 4; ++i)
                if (n16 / TP != wave) s_y[(4 * q + i) * LM + n16] = acc[i];  // (columns behind the block: zero)
    }
    float *out = a.ws + ((size_t)blockIdx.y * a.H + head) * scan_chunk_floats(SCAN_LINEAR, D);
    float *o_k = out + nblk * 256, *o_m = o_k + nblk * 256;
    for (int b = wave; b < nblk; b += 4) {
        dr_f32x4 r = *(const dr_f32x4 *)(s_r + n16 * LD + 16 * b + 4 * q), k;
        const dr_f32x4 l = *(const dr_f32x4 *)(s_l + max(n16 - 1, 0) * LD + 16 * b + 4 * q);
        const float l_end = s_l[(DC - 1) * LD + 16 * b + n16];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            r[i] *= n16 > 0 ? stack_exp<F32>(l[i]) : 1.0f;
            k[i] = s_k[(4 * q + i) * LD + 16 * b + n16] * stack_exp<F32>(l_end - s_l[(4 * q + i) * LD + 16 * b + n16]);
        }
        *(dr_f32x4 *)(out + b * 256 + lane * 4) = r, *(dr_f32x4 *)(o_k + b * 256 + lane * 4) = k;
    }
    if (wave == 1)
        for (int d = lane; d < 16 * nblk; d += 64) o_m[256 + d] = stack_exp<F32>(s_l[(DC - 1) * LD + d]);
    lds_barrier();
    if (wave == 0) *(dr_f32x4 *)(o_m + lane * 4) = *(const dr_f32x4 *)(s_y + n16 * LM + 4 * q);
}

size_t time_mix_prep_lds(int NB, int R8) {
    const size_t vec = (size_t)DC * (64 * NB + 4) * 4, low = (size_t)DC * (((R8 + 31) & ~31) + 8) * 4;
    return vec + DC * 20 * 4 + std::max(2 * vec, low);
}

template <class E, int NB>
int time_mix_chunks_nb(const TimeMixArgs &a, int chunks, hipStream_t st) {
    typedef typename E::type T;
    const size_t lds = time_mix_prep_lds(NB, a.R8);
    PIE_REQUIRE(lds <= 160 * 1024, PIE_E_SHAPE, "time mixing: head and decay rank too large together");
    static bool raised = false;
    if (!raised) {
        PIE_HIP_TRY(hipFuncSetAttribute((const void *)k_time_mix_prep<E, NB>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024));
        raised = true;
    }
    const ScanArgs scan = {(const T *)a.v, nullptr, a.ld, a.H, a.D, a.D, a.D8, a.pos, a.row_seq, a.slots, a.n_seqs, a.n_slots, a.runs, a.n_runs, a.state, a.slot_floats, a.ws, a.o, 0, 0};
    return scan_chunks<E, NB, SCAN_LINEAR>(scan, chunks, st, [&](int lo, int hi) {
        hipLaunchKernelGGL((k_time_mix_prep<E, NB>), dim3((unsigned)a.H, (unsigned)(hi - lo)), dim3(256), lds, st, a, lo);
    });
}
template <class E>
int time_mix_chunks_go(const TimeMixArgs &a, int chunks, hipStream_t st) {
    if (a.D <= 64) return time_mix_chunks_nb<E, 1>(a, chunks, st);
    if (a.D <= 128) return time_mix_chunks_nb<E, 2>(a, chunks, st);
    if (a.D <= 192) return time_mix_chunks_nb<E, 3>(a, chunks, st);
    return time_mix_chunks_nb<E, 4>(a, chunks, st);
}

template <class E>
int time_mix_step_go(const TimeMixArgs &a, hipStream_t st) {
    const dim3 grid((unsigned)a.n_runs, (unsigned)a.H, a.D <= 128 ? 1 : 2);
    const bool many = (long)a.n_runs * a.H > 256;
    if (a.D <= 64) hipLaunchKernelGGL((k_time_mix_step<E, 64, 512, 8>), grid, dim3(512), 0, st, a);
    else if (a.D <= 128 && many) hipLaunchKernelGGL((k_time_mix_step<E, 128, 512, 32>), grid, dim3(512), 0, st, a);
    else if (a.D <= 128) hipLaunchKernelGGL((k_time_mix_step<E, 128, 1024, 16>), grid, dim3(1024), 0, st, a);
    else hipLaunchKernelGGL((k_time_mix_step<E, 128, 1024, 32>), grid, dim3(1024), 0, st, a);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

int time_mix_check(const TimeMixArgs &a) {
    PIE_REQUIRE(a.D > 0 && a.D <= TIME_MIX_MAX_DIM && a.rank > 0 && a.rank <= TIME_MIX_MAX_RANK && a.H > 0 && a.H <= 65535, PIE_E_SHAPE,
                "time mixing: heads of at most 256 channels, decay rank of at most 1024");
    PIE_REQUIRE(a.slots && a.state && a.n_slots > 0, PIE_E_ARG, "time mixing: no state slots");
    return PIE_OK;
}

}  // namespace

size_t time_mix_ws_floats(int chunks, int H, int D) { return scan_ws_floats(SCAN_LINEAR, chunks, H, D); }
int time_mix_chunk_launches(int chunks, int H, int D) { return scan_launches(SCAN_LINEAR, chunks, H, D) + 1; }

static int time_mix_head_out(int dtype, const TimeMixArgs &a, int row0, int rows, hipStream_t st) {
    const HeadOutArgs h = {a.o, nullptr, a.gate, nullptr, a.ld, a.H, a.D, a.D8, a.o_norm, a.eps, a.out, a.ld_out, false, true, a.out_scale};
    return head_out_launch(dtype, h, row0, rows, st);
}

int time_mix_step_launch(int dtype, const TimeMixArgs &a, int row0, int rows, hipStream_t st) {
    if (a.n_runs <= 0) return PIE_OK;
    if (const int rc = time_mix_check(a)) return rc;
    PIE_REQUIRE(a.D <= 128 || a.o, PIE_E_ARG, "time mixing: wide heads need their output buffer");
    if (const int rc = dtype == PIE_F32 ? time_mix_step_go<ElemF32>(a, st) : time_mix_step_go<ElemBF16>(a, st)) return rc;
    return a.D > 128 ? time_mix_head_out(dtype, a, row0, rows, st) : PIE_OK;
}

int time_mix_chunks_launch(int dtype, const TimeMixArgs &a, int chunks, int row0, int rows, hipStream_t st) {
    if (a.n_runs <= 0) return PIE_OK;
    if (const int rc = time_mix_check(a)) return rc;
    PIE_REQUIRE(a.ws && a.o && chunks > 0 && a.n_runs <= 65535, PIE_E_ARG, "time mixing: the chunk form needs its workspace");
    if (const int rc = dtype == PIE_F32 ? time_mix_chunks_go<ElemF32>(a, chunks, st) : time_mix_chunks_go<ElemBF16>(a, chunks, st)) return rc;
    return time_mix_head_out(dtype, a, row0, rows, st);
}
