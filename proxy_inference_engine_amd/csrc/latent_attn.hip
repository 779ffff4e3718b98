// latent_attn.hip -- attention over a latent cache: every head scores the SAME cached vector c_j (R numbers per token) with its own query carried into
// the latent space (q' = W_uk^T q), and the softmax-weighted sum of the c_j is carried to values afterwards (W_uv per head).  Nothing but c is cached.
//
// For the matrix cores this is one [pairs x R] . [R x keys] product with pairs = (token, head): a workgroup takes up to 64 pairs of consecutive rows of
// one sequence -- a decoded token with its 32 heads, or a few tokens of a portion -- and a run of 32-key blocks (blockIdx.y: key split).  A block of
// latents is staged once in LDS and serves both products:
//   S^T[key, pair] = C . Q'^T         A = rows of C (ds_read_b128), B = the pairs' queries, kept in registers;
//   online softmax in fp32, base 2;   the reduction over keys runs over registers and two lane exchanges;
//   O^T[r, pair] += C^T . P^T         A = C^T by ds_read_b64_tr_b16, B = P^T as the score layout leaves it (the contraction runs over the keys in the
//                                     order 4 g + j, 16 + 4 g + j that both operands share), split into hi + lo bf16 halves: weights keep ~16 bits.
// Scores, weights, their sums and the accumulators are fp32.  A sliding window is a bound on i - j: blocks outside it are never read.
#include "stack_types.hpp"

typedef short v4s_t __attribute__((ext_vector_type(4)));
typedef __attribute__((ext_vector_type(8))) __bf16 la_bf16x8;
typedef __attribute__((ext_vector_type(4))) float la_f32x4;

namespace {

constexpr float LA_NEG = -1e30f, LA_LOG2E = 1.44269504088896340736f;
constexpr int LA_BK = 32;

__device__ __forceinline__ int la_page(const LatentAttnArgs &a, int seq, int t) {
    const int j = min(t / PAGE_TOKENS, a.table_width - 1);
    return (int)min((unsigned)a.table[(size_t)min(seq, a.n_seqs - 1) * a.table_width + j], (unsigned)a.n_pages - 1u);
}

template <int RC>
__device__ __forceinline__ int la_swizzle(int row) {
    const int sw = ((row & 3) << 2) | ((row >> 2) & 3);
    return RC % 2 ? sw & 7 : sw;
}
template <int RC>
__device__ __forceinline__ int la_off(int row, int ch) {  // byte offset of 16-byte chunk ch of key row: XOR-swizzled, conflict-free for both kinds of reads
    return row * (RC * 128) + 16 * (ch ^ la_swizzle<RC>(row));
}

// RC: latents of up to 64 RC numbers.  KH: key groups -- the four waves are 4 / KH tiles of 16 pairs times KH groups that take every KH-th block, so that a
// decoded token with few heads keeps all waves busy; the groups' sums meet in LDS at the end.
template <int RC, int KH>
__global__ void __launch_bounds__(256) k_latent_attn(const LatentAttnArgs a) {
    constexpr int PT = 4 / KH, PAIRS = 16 * PT;
    constexpr int BLOCK = LA_BK * RC * 128, ROUND = KH * BLOCK;  // bytes: a block of latents; what one round of the groups takes
    constexpr int NB = 2 * ROUND <= 128 * 1024 ? 2 : 1;          // two buffers (the next round lands while this one is multiplied) where they fit
    __shared__ __attribute__((aligned(1024))) char s_c[NB * ROUND];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int c = lane & 15, g = lane >> 4, pt = wave % PT, kg = wave / PT;
    int run_i = 0, pair0 = blockIdx.x;
    if (a.single) {
        const int per_run = (a.H + PAIRS - 1) / PAIRS;
        run_i = pair0 / per_run, pair0 %= per_run;
    } else {
        for (;;) {
            const int n = (a.runs[run_i].n_rows * a.H + PAIRS - 1) / PAIRS;
            if (pair0 < n || run_i + 1 >= a.n_runs) break;
            pair0 -= n, ++run_i;
        }
    }
    pair0 *= PAIRS;
    const RowRun tile = a.single ? RowRun{run_i, 1, a.row_seq[run_i], 0} : a.runs[run_i];
    const int last = min(PAIRS, tile.n_rows * a.H - pair0) - 1;
    if (last < 0) return;  // (a grid larger than the runs need)
    const int row_a = tile.row0 + pair0 / a.H, row_b = tile.row0 + (pair0 + last) / a.H;
    const int t_hi = a.pos[row_b], t_lo = a.window > 0 ? max(0, a.pos[row_a] - a.window + 1) : 0;
    const int nb = t_hi / LA_BK - t_lo / LA_BK + 1, per = ((nb + a.splits - 1) / a.splits + KH - 1) / KH * KH;
    const int b_begin = t_lo / LA_BK + (int)blockIdx.y * per, b_end = min(t_hi / LA_BK + 1, b_begin + per);

    // Blocks b .. b + KH - 1 into buffer `buf` by LDS-DMA, 1 KiB per wave instruction; the XOR swizzle is on the source side (LDS slot j of a row takes the
    // chunk that la_off maps there).  Chunks past the latent's end take the row's first one: the queries are zero there, and the sums are not stored.
    // Blocks behind the end repeat the last one; their group does not look at them.
    const unsigned lds0 = (unsigned)(size_t)(__attribute__((address_space(3))) void *)s_c;
    auto fetch = [&](int b, int buf) {
        unsigned long long src[KH];  // the blocks' first rows: wave-uniform, all looked up before the first DMA (a lookup between two would wait for the first)
#pragma unroll
        for (int k = 0; k < KH; ++k) {
            const int bb = min(b + k, b_end - 1);
            const unsigned long long v = (unsigned long long)(uintptr_t)((const u16 *)a.slab + ((size_t)la_page(a, tile.seq, bb * LA_BK) * PAGE_TOKENS + (bb & 1) * LA_BK) * a.ldr);
            src[k] = (unsigned long long)(unsigned)__builtin_amdgcn_readfirstlane((int)(unsigned)v) | ((unsigned long long)(unsigned)__builtin_amdgcn_readfirstlane((int)(unsigned)(v >> 32)) << 32);
        }
#pragma unroll
        for (int j = 0; j < KH * RC; ++j) {  // wave w moves rows of every block: instruction j = (block j / RC, KiB w RC + j % RC of it)
            const int k = j / RC, q = wave * RC + j % RC, x = q * 64 + lane, r = x / (8 * RC), ch = (x % (8 * RC)) ^ la_swizzle<RC>(r);
            const unsigned off = (unsigned)((r * a.ldr + (8 * ch < a.ldr ? 8 * ch : 0)) * 2), dst = lds0 + (unsigned)(buf * ROUND + k * BLOCK + q * 1024);
            unsigned keep;
            asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %3\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, %2\n\ts_mov_b32 m0, %0"
                         : "=&s"(keep)
                         : "v"(off), "s"(src[k]), "s"(dst)
                         : "memory");
        }
    };
    if (NB == 2 && b_begin < b_end) fetch(b_begin, 0);

    const bool busy = 16 * pt <= last;
    const int p = pair0 + min(16 * pt + c, last);
    const int row = tile.row0 + p / a.H, head = p % a.H;
    const size_t pr = (size_t)row * a.H + head;
    const int t_q = a.pos[row], t_min = a.window > 0 ? t_q - a.window + 1 : 0;
    const u16 *qp = (const u16 *)a.q + pr * a.ldr;
    uint4 qf[2 * RC];
#pragma unroll
    for (int s = 0; s < 2 * RC; ++s) qf[s] = 32 * s + 8 * g < a.ldr ? *(const uint4 *)(qp + 32 * s + 8 * g) : make_uint4(0, 0, 0, 0);

    la_f32x4 o[4 * RC];
#pragma unroll
    for (int r = 0; r < 4 * RC; ++r) o[r] = (la_f32x4){0.0f, 0.0f, 0.0f, 0.0f};
    float m_run = LA_NEG, l_run = 0.0f;
    const float sl2 = a.scale * LA_LOG2E;
    const int tq = (lane & 15) >> 2, tp = lane & 3;

    int buf = 0;
    bool started = false;
    for (int b = b_begin; b < b_end; b += KH) {
        if (NB == 1) {
            __syncthreads();
            fetch(b, 0);
        }
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();  // this round's blocks have landed for everyone, and nobody reads the other buffer any more
        const char *sb = s_c + buf * ROUND + kg * BLOCK;
        if (NB == 2) {
            if (b + KH < b_end) fetch(b + KH, buf ^ 1);
            buf ^= 1;
        }
        if (!busy || b + kg >= b_end) continue;
        // both products read LDS one batch ahead of their MFMAs (pinned: left alone the scheduler waits for every read at its use)
        constexpr int QB = (2 * RC) % 4 ? 2 : 4;
        la_f32x4 s0 = {0.0f, 0.0f, 0.0f, 0.0f}, s1 = s0, s2 = s0, s3 = s0;
        uint4 ka[2][QB], kb[2][QB];
        auto read_k = [&](int i, int slot) {
#pragma unroll
            for (int u = 0; u < QB; ++u) {
                ka[slot][u] = *(const uint4 *)(sb + la_off<RC>(c, 4 * (i * QB + u) + g));
                kb[slot][u] = *(const uint4 *)(sb + la_off<RC>(16 + c, 4 * (i * QB + u) + g));
            }
        };
        read_k(0, 0);
#pragma unroll
        for (int i = 0; i < 2 * RC / QB; ++i) {
            if (i + 1 < 2 * RC / QB) read_k(i + 1, (i + 1) & 1);
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int u = 0; u < QB; u += 2) {
                const la_bf16x8 qa = __builtin_bit_cast(la_bf16x8, qf[i * QB + u]), qb = __builtin_bit_cast(la_bf16x8, qf[i * QB + u + 1]);
                s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(la_bf16x8, ka[i & 1][u]), qa, s0, 0, 0, 0);
                s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(la_bf16x8, kb[i & 1][u]), qa, s1, 0, 0, 0);
                s2 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(la_bf16x8, ka[i & 1][u + 1]), qb, s2, 0, 0, 0);
                s3 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(la_bf16x8, kb[i & 1][u + 1]), qb, s3, 0, 0, 0);
            }
            __builtin_amdgcn_sched_barrier(0);
        }
        s0 += s2, s1 += s3;
        la_bf16x8 ct[2][4];
        auto read_c = [&](int i, int slot) {
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                const int ch = 2 * (4 * i + u) + (tp >> 1);
                const v4s_t a0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) v4s_t *)(sb + la_off<RC>(4 * g + tq, ch) + 8 * (tp & 1)));
                const v4s_t a1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) v4s_t *)(sb + la_off<RC>(16 + 4 * g + tq, ch) + 8 * (tp & 1)));
                const uint2 u0 = __builtin_bit_cast(uint2, a0), u1 = __builtin_bit_cast(uint2, a1);
                ct[slot][u] = __builtin_bit_cast(la_bf16x8, make_uint4(u0.x, u0.y, u1.x, u1.y));
            }
        };
        read_c(0, 0);
        __builtin_amdgcn_sched_barrier(0);
        // register i of s0 / s1 <-> key 32 (b + kg) + 4 g + i (+ 16)
        const int t0 = (b + kg) * LA_BK + 4 * g;
        float sc[8], mloc = LA_NEG;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const int t = t0 + (i & 3) + 16 * (i >> 2);
            sc[i] = (t <= t_q && t >= t_min) ? (i < 4 ? s0[i & 3] : s1[i & 3]) * sl2 : LA_NEG;
            mloc = fmaxf(mloc, sc[i]);
        }
        mloc = xor32_max(xor16_max(mloc));
        // The running maximum moves only when a score exceeds it by 2^8 (weights of up to 256 are as exact as weights of up to 1): rescaling is rare.
        if (!started) m_run = mloc, started = true;
        else if (__builtin_amdgcn_ballot_w64(mloc > m_run + 8.0f)) {
            const float mm = fmaxf(m_run, mloc), alpha = __builtin_amdgcn_exp2f(m_run - mm);
            l_run *= alpha;
#pragma unroll
            for (int r = 0; r < 4 * RC; ++r) o[r] *= alpha;
            m_run = mm;
        }
        u32 hi[4], lo[4];
#pragma unroll
        for (int i = 0; i < 8; i += 2) {
            const float pa = sc[i] > LA_NEG ? __builtin_amdgcn_exp2f(sc[i] - m_run) : 0.0f, pb = sc[i + 1] > LA_NEG ? __builtin_amdgcn_exp2f(sc[i + 1] - m_run) : 0.0f;
            l_run += pa + pb;
            const float ha = round_T<BF16>(pa), hb = round_T<BF16>(pb);
            hi[i >> 1] = pack2<BF16>(ha, hb);
            lo[i >> 1] = pack2<BF16>(pa - ha, pb - hb);
        }
        const la_bf16x8 ph = __builtin_bit_cast(la_bf16x8, make_uint4(hi[0], hi[1], hi[2], hi[3]));
        const la_bf16x8 pl = __builtin_bit_cast(la_bf16x8, make_uint4(lo[0], lo[1], lo[2], lo[3]));
#pragma unroll
        for (int i = 0; i < RC; ++i) {
            if (i + 1 < RC) read_c(i + 1, (i + 1) & 1);
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int u = 0; u < 4; ++u) o[4 * i + u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ct[i & 1][u], ph, o[4 * i + u], 0, 0, 0);
#pragma unroll
            for (int u = 0; u < 4; ++u) o[4 * i + u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ct[i & 1][u], pl, o[4 * i + u], 0, 0, 0);
            __builtin_amdgcn_sched_barrier(0);
        }
    }
    float l = xor32_sum(xor16_sum(l_run));
    if constexpr (KH > 1) {  // merge the key groups, halving: group kg + half hands its sums to group kg through LDS (16 pairs x 64 RC floats per pair tile)
        __shared__ float s_ml[4][16][2];
#pragma unroll
        for (int half = KH / 2; half >= 1; half >>= 1) {
            __syncthreads();
            float *so = (float *)s_c + ((size_t)(kg % half) * PT + pt) * 16 * 64 * RC;
            if (kg >= half && kg < 2 * half) {
#pragma unroll
                for (int r = 0; r < 4 * RC; ++r) *(la_f32x4 *)(so + (r * 64 + lane) * 4) = o[r];
                if (g == 0) s_ml[wave - half * PT][c][0] = m_run, s_ml[wave - half * PT][c][1] = l;
            }
            __syncthreads();
            if (kg < half) {
                const float m2 = s_ml[wave][c][0], l2 = s_ml[wave][c][1], mm = fmaxf(m_run, m2);
                const float f1 = __builtin_amdgcn_exp2f(m_run - mm), f2 = __builtin_amdgcn_exp2f(m2 - mm);
#pragma unroll
                for (int r = 0; r < 4 * RC; ++r) {
                    const la_f32x4 v = *(const la_f32x4 *)(so + (r * 64 + lane) * 4);
#pragma unroll
                    for (int i = 0; i < 4; ++i) o[r][i] = fmaf(f2, v[i], f1 * o[r][i]);
                }
                l = l * f1 + l2 * f2, m_run = mm;
            }
        }
    }
    if (kg > 0 || 16 * pt + c > last) return;
    const size_t MH = (size_t)a.M * a.H;
    if (a.splits == 1) {
        const float inv = 1.0f / l;
        u16 *dst = (u16 *)a.out + pr * a.ldr;
#pragma unroll
        for (int r = 0; r < 4 * RC; ++r)
            if (16 * r + 4 * g < a.ldr)
                *(uint2 *)(dst + 16 * r + 4 * g) = make_uint2(pack2<BF16>(o[r][0] * inv, o[r][1] * inv), pack2<BF16>(o[r][2] * inv, o[r][3] * inv));
    } else {
        float *dst = a.ws + ((size_t)blockIdx.y * MH + pr) * a.ldr;
        if (l > 0.0f)
#pragma unroll
            for (int r = 0; r < 4 * RC; ++r)
                if (16 * r + 4 * g < a.ldr) *(la_f32x4 *)(dst + 16 * r + 4 * g) = o[r];
        if (g == 0) {
            float *ml = a.ws + (size_t)a.splits * MH * a.ldr + ((size_t)blockIdx.y * MH + pr) * 2;
            ml[0] = m_run, ml[1] = l;
        }
    }
}

// merges the key splits of one (token, head) pair: every wave weighs all splits (at most 64: one per lane), then streams the partial sums, eight in flight
__global__ void __launch_bounds__(128) k_latent_combine(const LatentAttnArgs a) {
    __shared__ float s_f[64];
    const size_t pr = blockIdx.x, MH = (size_t)a.M * a.H;
    const int lane = threadIdx.x & 63;
    const float2 ml = lane < a.splits ? *(const float2 *)(a.ws + (size_t)a.splits * MH * a.ldr + (lane * MH + pr) * 2) : make_float2(LA_NEG, 0.0f);
    const float m = wave_max(ml.y > 0.0f ? ml.x : LA_NEG);
    const float f = ml.y > 0.0f ? __builtin_amdgcn_exp2f(ml.x - m) : 0.0f;  // an empty split wrote no sums and has no weight
    const float l = wave_sum(ml.y * f);
    if (threadIdx.x < 64) s_f[lane] = f / l;
    __syncthreads();
    for (int r = threadIdx.x * 4; r < a.ldr; r += 512) {
        la_f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
        for (int s0 = 0; s0 < a.splits; s0 += 8) {
            la_f32x4 v[8];
            float w[8];
#pragma unroll
            for (int u = 0; u < 8; ++u) {
                const int s = min(s0 + u, a.splits - 1);
                w[u] = s0 + u < a.splits ? s_f[s] : 0.0f;
                v[u] = *(const la_f32x4 *)(a.ws + (s * MH + pr) * a.ldr + r);
            }
#pragma unroll
            for (int u = 0; u < 8; ++u)
#pragma unroll
                for (int i = 0; i < 4; ++i) acc[i] = w[u] > 0.0f ? fmaf(w[u], v[u][i], acc[i]) : acc[i];
        }
        *(uint2 *)((u16 *)a.out + pr * a.ldr + r) = make_uint2(pack2<BF16>(acc[0], acc[1]), pack2<BF16>(acc[2], acc[3]));
    }
}

// One (row, head) per workgroup on the vector ALU: fp32 stacks, and latents wider than the MFMA kernel's registers hold.
constexpr int LA_RMAX = 2048;
template <class E>
__global__ void __launch_bounds__(256) k_latent_attn_rows(const LatentAttnArgs a) {
    typedef typename E::type T;
    __shared__ float s_o[4][LA_RMAX], s_q[LA_RMAX], s_m[4], s_l[4];
    const int row = blockIdx.x, head = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const size_t pr = (size_t)row * a.H + head;
    for (int r = threadIdx.x; r < a.R; r += 256) s_q[r] = E::load((const T *)a.q + pr * a.ldr + r);
    for (int r = lane; r < a.R; r += 64) s_o[wave][r] = 0.0f;
    __syncthreads();
    const int t_q = a.pos[row], t_lo = a.window > 0 ? max(0, t_q - a.window + 1) : 0, seq = a.row_seq[row];
    float m = LA_NEG, l = 0.0f;
    for (int t = t_lo + wave; t <= t_q; t += 4) {
        const T *cp = (const T *)a.slab + ((size_t)la_page(a, seq, t) * PAGE_TOKENS + (t & (PAGE_TOKENS - 1))) * a.ldr;
        float d = 0.0f;
        for (int r = lane; r < a.R; r += 64) d = fmaf(s_q[r], E::load(cp + r), d);
        d = wave_sum(d) * a.scale;
        const float m2 = fmaxf(m, d), f = expf(m - m2), w = expf(d - m2);
        l = l * f + w, m = m2;
        for (int r = lane; r < a.R; r += 64) s_o[wave][r] = fmaf(w, E::load(cp + r), s_o[wave][r] * f);
    }
    if (lane == 0) s_m[wave] = m, s_l[wave] = l;
    __syncthreads();
    const float mx = fmaxf(fmaxf(s_m[0], s_m[1]), fmaxf(s_m[2], s_m[3]));
    float f[4], sum = 0.0f;
#pragma unroll
    for (int w = 0; w < 4; ++w) f[w] = s_l[w] > 0.0f ? expf(s_m[w] - mx) : 0.0f, sum += s_l[w] * f[w];
    for (int r = threadIdx.x; r < a.R; r += 256)
        ((T *)a.out)[pr * a.ldr + r] = E::pack((s_o[0][r] * f[0] + s_o[1][r] * f[1] + s_o[2][r] * f[2] + s_o[3][r] * f[3]) / sum);
}

template <class E, class X>
__global__ void __launch_bounds__(256) k_latent_append(const typename X::type *c_raw, int ldc, const float *w, float eps, int R, int ldr, const int *pos, const int *row_seq,
                                                       const int *table, int table_width, int n_pages, int n_seqs, typename E::type *slab) {
    __shared__ float red[4];
    const int m = blockIdx.x;
    const typename X::type *x = c_raw + (size_t)m * ldc;
    float ss = 0.0f;
    for (int r = threadIdx.x; r < R; r += 256) {
        const float v = X::load(x + r);
        ss = fmaf(v, v, ss);
    }
    ss = wave_sum(ss);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    const float inv = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)R + eps);
    const int t = pos[m], j = min(t / PAGE_TOKENS, table_width - 1);
    const size_t page = min((unsigned)table[(size_t)min(row_seq[m], n_seqs - 1) * table_width + j], (unsigned)n_pages - 1u);
    typename E::type *dst = slab + (page * PAGE_TOKENS + (t & (PAGE_TOKENS - 1))) * ldr;
    for (int r = threadIdx.x; r < R; r += 256) dst[r] = E::pack(X::load(x + r) * inv * w[r]);
}

}  // namespace

int latent_attn_pairs(int H, int R, bool single) {
    if (!single || R > 512) return 64;
    return H <= 16 ? 16 : H <= 32 ? 32 : 64;
}

size_t latent_attn_ws_floats(int M, int H, int R, int splits) { return splits > 1 ? (size_t)splits * M * H * (((R + 7) & ~7) + 2) : 0; }

int latent_attn_launch(int dtype, const LatentAttnArgs &a, hipStream_t st) {
    if (a.M <= 0) return PIE_OK;
    PIE_REQUIRE(a.R > 0 && a.R <= LA_RMAX && a.H > 0 && a.H <= 65535, PIE_E_SHAPE, "latent attention: kv_rank must be 1 .. 2048");
    PIE_REQUIRE(a.splits >= 1 && (a.splits == 1 || a.ws), PIE_E_ARG, "latent attention: a key split needs its workspace");
    if (dtype == PIE_F32 || a.R > 1024) {
        const dim3 grid((unsigned)a.M, (unsigned)a.H);
        if (dtype == PIE_F32) hipLaunchKernelGGL(k_latent_attn_rows<ElemF32>, grid, dim3(256), 0, st, a);
        else hipLaunchKernelGGL(k_latent_attn_rows<ElemBF16>, grid, dim3(256), 0, st, a);
        PIE_LAUNCH_CHECK();
        return PIE_OK;
    }
    if (a.n_tiles <= 0) return PIE_OK;
    const dim3 grid((unsigned)a.n_tiles, (unsigned)a.splits);
    const int rc = (a.R + 63) / 64;
#define LA_GO(N) \
    if (a.pairs == 16) hipLaunchKernelGGL((k_latent_attn<N, 4>), grid, dim3(256), 0, st, a); \
    else if (a.pairs == 32) hipLaunchKernelGGL((k_latent_attn<N, 2>), grid, dim3(256), 0, st, a); \
    else hipLaunchKernelGGL((k_latent_attn<N, 1>), grid, dim3(256), 0, st, a)
    if (rc <= 1) { LA_GO(1); }
    else if (rc <= 2) { LA_GO(2); }
    else if (rc <= 3) { LA_GO(3); }
    else if (rc <= 4) { LA_GO(4); }
    else if (rc <= 6) { LA_GO(6); }
    else if (rc <= 8) { LA_GO(8); }
    else if (rc <= 10) hipLaunchKernelGGL((k_latent_attn<10, 1>), grid, dim3(256), 0, st, a);
    else hipLaunchKernelGGL((k_latent_attn<16, 1>), grid, dim3(256), 0, st, a);
#undef LA_GO
    PIE_LAUNCH_CHECK();
    if (a.splits > 1) {
        hipLaunchKernelGGL(k_latent_combine, dim3((unsigned)(a.M * a.H)), dim3(128), 0, st, a);
        PIE_LAUNCH_CHECK();
    }
    return PIE_OK;
}

int latent_append_launch(int dtype, const void *c_raw, bool raw16, int ldc, const float *w, float eps, int M, int R, int ldr, const int *pos, const int *row_seq,
                         const int *table, int table_width, int n_pages, int n_seqs, void *slab, hipStream_t st) {
    if (M <= 0) return PIE_OK;
#define APPEND_GO(E_, X_) \
    hipLaunchKernelGGL((k_latent_append<E_, X_>), dim3((unsigned)M), dim3(256), 0, st, (const X_::type *)c_raw, ldc, w, eps, R, ldr, pos, row_seq, table, table_width, n_pages, \
                       n_seqs, (E_::type *)slab)
    if (dtype == PIE_F32) APPEND_GO(ElemF32, ElemF32);
    else if (raw16) APPEND_GO(ElemBF16, ElemBF16);
    else APPEND_GO(ElemBF16, ElemF32);
#undef APPEND_GO
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}
