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
// leaves T U, R, K, -A and T A, A', -B' in matrix operand order; a second walks the chunks (chunk_scan.hpp, SCAN_DELTA); a third takes the heads' norm and gate.  W_16 is
// above exp(-16 decay_scale): the quotients are formed as W_t times 1 / W_i, which fp32 holds up to DELTA_MAX_DECAY.
#include "chunk_scan.hpp"
#include "low_rank.hpp"

namespace {

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
    const ScanChunk c = scan_chunk(a.runs, a.n_runs, a.chunk_lo + (int)blockIdx.y);
    if (c.n <= 0) return;
    typedef ElemPair Pair;
    auto bias_at = [&](int at) -> Pair {
        if (!a.bias) return {0.0f, 0.0f};
        const u32 w = *(const u32 *)(a.bias + at);
        return {lo_f32<BF16>(w), hi_f32<BF16>(w)};
    };
    // All loads without branches around them: they leave together, and what lies outside is dropped afterwards.
    const T *raw = (const T *)a.raw + (size_t)c.row0 * a.ld;
    const LowRankArgs low = {raw + 5 * HD8, a.ld, c.n, a.rank, a.R8, a.bias ? a.bias + 5 * HD8 : nullptr, a.w_decay + (size_t)head * D * a.R8, a.decay_bias + head * D, D};
    LowRank<E, NB> lr;
    lr.load(low);
    Pair xr[NP][TP], xk[NP][TP], xa[NP][TP], bx[NP][3];
#pragma unroll
    for (int p = 0; p < NP; ++p) {
        const int d = min(2 * (lane + 64 * p), a.D8 - 2) + head * a.D8;  // (heads are padded to a multiple of 8)
#pragma unroll
        for (int j = 0; j < TP; ++j) {
            const T *x = raw + (size_t)min(TP * wave + j, c.n - 1) * a.ld;
            xr[p][j] = load_pair<E>(x + d), xk[p][j] = load_pair<E>(x + HD8 + d), xa[p][j] = load_pair<E>(x + 4 * HD8 + d);
        }
        bx[p][0] = bias_at(d), bx[p][1] = bias_at(HD8 + d), bx[p][2] = bias_at(4 * HD8 + d);
    }
    lr.load_weights(low, wave, lane);
    lr.put(low, s_u);
    lds_barrier();
    lr.product(low, s_u, wave, lane, [&](int t, int d, float z) { s_l[t * LD + d] = t < c.n && d < D ? -a.decay_scale * stack_sigmoid<F32>(z) : 0.0f; });
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
    float *out = a.ws + ((size_t)blockIdx.y * a.H + head) * scan_chunk_floats(SCAN_DELTA, D);
    float *o_r = out + nblk * 256, *o_k = o_r + nblk * 256, *o_a = o_k + nblk * 256, *o_m = o_a + nblk * 256;
    float *s_t = s_m + 4 * DC * LM;
    if (wave == 0) {
        float tc[DC];
        scan_inverse<LM>(s_m + DC * LM, n16, tc);
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
    const int v0 = 2 * a.H * a.D8;
    const ScanArgs scan = {(const typename E::type *)a.raw + v0, a.bias ? a.bias + v0 : nullptr, a.ld, a.H, a.D, a.D, a.D8, a.pos, a.row_seq, a.slots, a.n_seqs, a.n_slots, a.runs, a.n_runs, a.state,
                           a.slot_floats, a.ws, a.o, 0, 0};
    const int rc = scan_chunks<E, NB, SCAN_DELTA>(scan, chunks, st, [&](int lo, int hi) {
        seg.chunk_lo = lo, seg.chunk_hi = hi;
        hipLaunchKernelGGL((k_delta_prep<E, NB>), dim3((unsigned)a.H, (unsigned)(hi - lo)), dim3(256), lds, st, seg);
    });
    if (rc) return rc;
    const int g0 = 3 * a.H * a.D8;
    const HeadOutArgs h = {a.o, nullptr, (const typename E::type *)a.raw + g0, a.bias ? a.bias + g0 : nullptr, a.ld, a.H, a.D, a.D8, a.o_norm, a.eps, a.out, a.ld_out, false, false, 1.0f};
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
size_t delta_ws_floats(int chunks, int H, int D) { return scan_ws_floats(SCAN_DELTA, chunks, H, D); }
int delta_launches(int chunks, int H, int D) { return scan_launches(SCAN_DELTA, chunks, H, D) + 1; }

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
