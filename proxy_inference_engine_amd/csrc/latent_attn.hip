// latent_attn.hip -- attention over a latent cache: every head scores the SAME cached vector c_j (R numbers per token) with its own query carried into
// the latent space (q' = W_uk^T q), and the softmax-weighted sum of the c_j is carried to values afterwards (W_uv per head).  Nothing but c is cached.
//
// For the matrix cores this is one [pairs x R] . [R x keys] product with pairs = (token, head): a workgroup takes up to 32 pairs of consecutive rows of
// one sequence -- a decoded token with its 32 heads, or a few tokens of a portion -- and a run of 32-key blocks (blockIdx.y: key split).  A block of
// latents is staged once in LDS and serves both products:
//   S^T[key, pair] = C . Q'^T         A = rows of C (ds_read_b128), B = the pairs' queries, kept in registers;
//   online softmax in fp32, base 2;   the reduction over keys runs over registers and one lane exchange;
//   O^T[r, pair] += C^T . P^T         (r: the latent's own numbers) A = C^T by ds_read_b64_tr_b16, B = P^T as the score layout leaves it, split into hi + lo bf16 halves: weights
//                                     keep ~16 bits.
// A cached row may hold more than the latent: numbers behind it that scores read too (a rotated key part all heads share), against a second part of the queries.
// Where the sums are finished the denominator takes the head's sink, and the result the head's gate.
// Scores, weights, their sums and the accumulators are fp32.  A sliding window is a bound on i - j: blocks outside it are never read.
#include "mfma_store.hpp"    // w4m_pack
#include "prefill_attn.hpp"  // MfmaT, f32x16_t
#include "stack_types.hpp"

typedef short v4s_t __attribute__((ext_vector_type(4)));
typedef __attribute__((ext_vector_type(4))) float la_f32x4;

namespace {

constexpr float LA_NEG = -1e30f, LA_LOG2E = 1.44269504088896340736f;
constexpr int LA_BK = 32, LA_PAIRS = 32;

__device__ __forceinline__ int la_page(const LatentAttnArgs &a, int seq, int t) {
    const int j = min(t / PAGE_TOKENS, a.table_width - 1);
    return (int)min((unsigned)a.table[(size_t)min(seq, a.n_seqs - 1) * a.table_width + j], (unsigned)a.n_pages - 1u);
}

__device__ __forceinline__ int la_swizzle(int row) { return ((row & 3) << 2) | ((row >> 2) & 3); }
template <int RC>
__device__ __forceinline__ int la_off(int row, int ch) {  // byte offset of 16-byte chunk ch of key row: XOR-swizzled, conflict-free for both kinds of reads
    return row * (RC * 128) + 16 * (ch ^ la_swizzle(row));
}

// RC: latents of up to 64 RC numbers (even).  A workgroup's 32 pairs are one column block of v_mfma_f32_32x32x16; its four waves split the LATENT: each owns
// R / 4 columns of C, for which it takes a partial score product (the four partials are added through LDS, in wave order, by every wave: all hold the
// same scores and weights) and its own quarter of the weighted sums.  So every staged number is read from LDS once per product, and a wave keeps only a
// quarter of the queries and accumulators in registers.
template <int RC>
__global__ void __launch_bounds__(256, RC <= 8 ? 2 : 1) k_latent_attn(const LatentAttnArgs a) {
    constexpr int BLOCK = LA_BK * RC * 128, NB = 2;  // bytes of a block of latents; buffers (more measured no faster: two workgroups per CU cover the latency)
    __shared__ __attribute__((aligned(1024))) char s_c[NB * BLOCK];
    __shared__ __attribute__((aligned(16))) float s_part[4][4][64][4];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int c = lane & 31, h = lane >> 5;
    int run_i = 0, pair0 = blockIdx.x;
    if (a.single) {
        const int per_run = (a.H + LA_PAIRS - 1) / LA_PAIRS;
        run_i = pair0 / per_run, pair0 %= per_run;
    } else {
        for (;;) {
            const int n = (a.runs[run_i].n_rows * a.H + LA_PAIRS - 1) / LA_PAIRS;
            if (pair0 < n || run_i + 1 >= a.n_runs) break;
            pair0 -= n, ++run_i;
        }
    }
    pair0 *= LA_PAIRS;
    const RowRun tile = a.single ? RowRun{run_i, 1, a.row_seq[run_i], 0} : a.runs[run_i];
    const int last = min(LA_PAIRS, tile.n_rows * a.H - pair0) - 1;
    if (last < 0) return;  // (a grid larger than the runs need)
    const int row_a = tile.row0 + pair0 / a.H, row_b = tile.row0 + (pair0 + last) / a.H;
    const int t_hi = a.pos[row_b], t_lo = a.window > 0 ? max(0, a.pos[row_a] - a.window + 1) : 0;
    const int nb = t_hi / LA_BK - t_lo / LA_BK + 1, per = (nb + a.splits - 1) / a.splits;
    const int b_begin = t_lo / LA_BK + (int)blockIdx.y * per, b_end = min(t_hi / LA_BK + 1, b_begin + per);

    // Block b into buffer `buf` by LDS-DMA, 1 KiB per wave instruction; the XOR swizzle is on the source side (LDS slot j of a row takes the chunk that
    // la_off maps there).  Chunks past the latent's end take the row's first one: the queries are zero there, and the sums are not stored.  Blocks behind
    // the end repeat the last one.  Pages come from registers: a lookup in memory would wait for the DMAs before it.
    const unsigned lds0 = (unsigned)(size_t)(__attribute__((address_space(3))) void *)s_c;
    int pg_first = b_begin / 2, pg = la_page(a, tile.seq, (pg_first + lane) * PAGE_TOKENS);  // lane l: the page of blocks 2 (pg_first + l), + 1
    auto fetch = [&](int b, int buf) {
        const int bb = min(b, b_end - 1);
        int i = bb / 2 - pg_first;
        if (i >= 64) pg_first = bb / 2, i = 0, pg = la_page(a, tile.seq, (pg_first + lane) * PAGE_TOKENS);
        const unsigned long long v = (unsigned long long)(uintptr_t)((const u16 *)a.slab + ((size_t)__builtin_amdgcn_readlane(pg, i) * PAGE_TOKENS + (bb & 1) * LA_BK) * a.ldr);
        const unsigned long long src =
            (unsigned long long)(unsigned)__builtin_amdgcn_readfirstlane((int)(unsigned)v) | ((unsigned long long)(unsigned)__builtin_amdgcn_readfirstlane((int)(unsigned)(v >> 32)) << 32);
#pragma unroll
        for (int j = 0; j < RC; ++j) {
            const int q = wave * RC + j, x = q * 64 + lane, r = x / (8 * RC), ch = (x % (8 * RC)) ^ la_swizzle(r);
            const unsigned off = (unsigned)((r * a.ldr + (8 * ch < a.ldr ? 8 * ch : 0)) * 2), dst = lds0 + (unsigned)(buf * BLOCK + q * 1024);
            unsigned keep;
            asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %3\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, %2\n\ts_mov_b32 m0, %0"
                         : "=&s"(keep)
                         : "v"(off), "s"(src), "s"(dst)
                         : "memory");
        }
    };
    if (b_begin < b_end)
#pragma unroll
        for (int i = 0; i < NB - 1; ++i) fetch(b_begin + i, i);  // (blocks behind the end repeat the last one: the wait below counts instructions)

    const int p = pair0 + min(c, last);
    const int row = tile.row0 + p / a.H, head = p % a.H;
    const size_t pr = (size_t)row * a.H + head;
    const int t_q = a.pos[row], t_min = a.window > 0 ? t_q - a.window + 1 : 0;
    const int col0 = 16 * RC * wave;  // the wave's columns of the latent
    uint4 qf[RC];
#pragma unroll
    for (int s = 0; s < RC; ++s) {
        const int at = col0 + 16 * s + 8 * h;
        const u16 *qp = (const u16 *)a.q + pr * a.ldq + at;
        if (at >= a.ldq) qp = (const u16 *)a.q_rot + (size_t)row * a.ld_rot + head * (a.ldr - a.ldq) + at - a.ldq;
        qf[s] = at < a.ldr ? *(const uint4 *)qp : make_uint4(0, 0, 0, 0);
    }

    f32x16_t o[RC / 2];
#pragma unroll
    for (int d = 0; d < RC / 2; ++d)
#pragma unroll
        for (int i = 0; i < 16; ++i) o[d][i] = 0.0f;
    float m_run = LA_NEG, l_run = 0.0f;
    const float sl2 = a.scale * LA_LOG2E;
    const int grp = lane >> 4, tq = (lane & 15) >> 2, tp = lane & 3;
    bool started = false;
    int buf = 0;

    for (int b = b_begin; b < b_end; ++b) {
        asm volatile("s_waitcnt vmcnt(%0)" ::"n"((NB - 2) * RC) : "memory");
        __syncthreads();  // this block has landed for everyone; nobody reads the oldest buffer or the partial scores any more
        fetch(b + NB - 1, buf ? buf - 1 : NB - 1);
        const char *sb = s_c + buf * BLOCK;
        buf = buf + 1 < NB ? buf + 1 : 0;
        f32x16_t s0;
#pragma unroll
        for (int i = 0; i < 16; ++i) s0[i] = 0.0f;
        {
            uint4 k[RC];
#pragma unroll
            for (int s = 0; s < RC; ++s) k[s] = *(const uint4 *)(sb + la_off<RC>(c, 2 * RC * wave + 2 * s + h));
            __builtin_amdgcn_sched_barrier(0);  // all reads in flight before the first product
#pragma unroll
            for (int s = 0; s < RC; ++s) s0 = MfmaT<BF16>::run(k[s], qf[s], s0);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) *(la_f32x4 *)s_part[wave][i][lane] = (la_f32x4){s0[4 * i], s0[4 * i + 1], s0[4 * i + 2], s0[4 * i + 3]};
        __syncthreads();
        // the weighted sums' first operands are on their way while the scores are added up
        uint4 ct[2][2];
        auto read_c = [&](int s, int d) {
            const int ch = 2 * RC * wave + 4 * d + 2 * (grp & 1) + (tp >> 1);
            const v4s_t a0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) v4s_t *)(sb + la_off<RC>(16 * s + 4 * h + tq, ch) + 8 * (tp & 1)));
            const v4s_t a1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) v4s_t *)(sb + la_off<RC>(16 * s + 8 + 4 * h + tq, ch) + 8 * (tp & 1)));
            const uint2 u0 = __builtin_bit_cast(uint2, a0), u1 = __builtin_bit_cast(uint2, a1);
            return make_uint4(u0.x, u0.y, u1.x, u1.y);
        };
        float sc[16], mloc = LA_NEG;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const la_f32x4 w0 = *(const la_f32x4 *)s_part[0][i][lane], w1 = *(const la_f32x4 *)s_part[1][i][lane];
            const la_f32x4 w2 = *(const la_f32x4 *)s_part[2][i][lane], w3 = *(const la_f32x4 *)s_part[3][i][lane];
#pragma unroll
            for (int j = 0; j < 4; ++j) sc[4 * i + j] = ((w0[j] + w1[j]) + (w2[j] + w3[j])) * sl2;
        }
        ct[0][0] = read_c(0, 0), ct[0][1] = read_c(1, 0);
        // register i <-> key 32 b + (i & 3) + 8 (i >> 2) + 4 h
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const int t = b * LA_BK + (i & 3) + 8 * (i >> 2) + 4 * h;
            sc[i] = t <= t_q && t >= t_min ? sc[i] : LA_NEG;
            mloc = fmaxf(mloc, sc[i]);
        }
        mloc = xor32_max(mloc);
        // The running maximum moves only when a score exceeds it by 2^8 (weights of up to 256 are as exact as weights of up to 1): rescaling is rare.
        if (!started) m_run = mloc, started = true;
        else if (__builtin_amdgcn_ballot_w64(mloc > m_run + 8.0f)) {
            const float mm = fmaxf(m_run, mloc), alpha = __builtin_amdgcn_exp2f(m_run - mm);
            l_run *= alpha;
#pragma unroll
            for (int d = 0; d < RC / 2; ++d)
#pragma unroll
                for (int i = 0; i < 16; ++i) o[d][i] *= alpha;
            m_run = mm;
        }
        u32 hi[8], lo[8];
#pragma unroll
        for (int i = 0; i < 16; i += 2) {
            const float pa = sc[i] > LA_NEG ? __builtin_amdgcn_exp2f(sc[i] - m_run) : 0.0f, pb = sc[i + 1] > LA_NEG ? __builtin_amdgcn_exp2f(sc[i + 1] - m_run) : 0.0f;
            l_run += pa + pb;
            const u32 w = w4m_pack<BF16>(pa, pb);
            hi[i >> 1] = w;
            lo[i >> 1] = w4m_pack<BF16>(pa - lo_f32<BF16>(w), pb - hi_f32<BF16>(w));
        }
#pragma unroll
        for (int d = 0; d < RC / 2; ++d) {
            if (col0 + 32 * d >= a.ldq) break;  // (wave-uniform: nothing but score numbers, or nothing at all)
            if (d + 1 < RC / 2) ct[(d + 1) & 1][0] = read_c(0, d + 1), ct[(d + 1) & 1][1] = read_c(1, d + 1);
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int s = 0; s < 2; ++s) {
                o[d] = MfmaT<BF16>::run(ct[d & 1][s], make_uint4(hi[4 * s], hi[4 * s + 1], hi[4 * s + 2], hi[4 * s + 3]), o[d]);
                o[d] = MfmaT<BF16>::run(ct[d & 1][s], make_uint4(lo[4 * s], lo[4 * s + 1], lo[4 * s + 2], lo[4 * s + 3]), o[d]);
            }
            __builtin_amdgcn_sched_barrier(0);
        }
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // the look-ahead DMAs: LDS is handed on when the workgroup ends
    const float l = xor32_sum(l_run);
    if (c > last) return;
    const size_t MH = (size_t)a.M * a.H;
    if (a.splits == 1) {
        const float inv = head_gate<false>(a.finish, row, head) / (l + head_sink2(a.finish, head, m_run));
        u16 *dst = (u16 *)a.out + pr * a.ldq + col0;
#pragma unroll
        for (int d = 0; d < RC / 2; ++d)
#pragma unroll
            for (int k = 0; k < 4; ++k)  // registers 4k .. 4k + 3 <-> columns 32 d + 8 k + 4 h + {0..3}
                if (col0 + 32 * d + 8 * k + 4 * h < a.ldq)
                    *(uint2 *)(dst + 32 * d + 8 * k + 4 * h) =
                        make_uint2(w4m_pack<BF16>(o[d][4 * k] * inv, o[d][4 * k + 1] * inv), w4m_pack<BF16>(o[d][4 * k + 2] * inv, o[d][4 * k + 3] * inv));
    } else {
        float *dst = a.ws + ((size_t)blockIdx.y * MH + pr) * a.ldq + col0;
        if (l > 0.0f)
#pragma unroll
            for (int d = 0; d < RC / 2; ++d)
#pragma unroll
                for (int k = 0; k < 4; ++k)
                    if (col0 + 32 * d + 8 * k + 4 * h < a.ldq)
                        *(la_f32x4 *)(dst + 32 * d + 8 * k + 4 * h) = (la_f32x4){o[d][4 * k], o[d][4 * k + 1], o[d][4 * k + 2], o[d][4 * k + 3]};
        if (wave == 0 && h == 0) {
            float *ml = a.ws + (size_t)a.splits * MH * a.ldq + ((size_t)blockIdx.y * MH + pr) * 2;
            ml[0] = m_run, ml[1] = l;
        }
    }
}

// merges the key splits of one (token, head) pair
__global__ void __launch_bounds__(128) k_latent_combine(const LatentMerge a, u16 *out) {
    __shared__ float s_f[64];
    const size_t pr = blockIdx.x;
    const float f = latent_split_weight(a, pr, threadIdx.x & 63);
    if (threadIdx.x < 64) s_f[threadIdx.x] = f;
    __syncthreads();
    for (int r = threadIdx.x * 4; r < a.ldr; r += 512) {
        const float4 v = latent_merge4(a, pr, r, [&](int s) { return s_f[s]; });
        *(uint2 *)(out + pr * a.ldr + r) = make_uint2(pack2<BF16>(v.x, v.y), pack2<BF16>(v.z, v.w));
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
    for (int r = threadIdx.x; r < a.R; r += 256)
        s_q[r] = E::load(r < a.ldq ? (const T *)a.q + pr * a.ldq + r : (const T *)a.q_rot + (size_t)row * a.ld_rot + head * (a.ldr - a.ldq) + r - a.ldq);
    const int RO = min(a.R, a.ldq);
    for (int r = lane; r < RO; r += 64) s_o[wave][r] = 0.0f;
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
        for (int r = lane; r < RO; r += 64) s_o[wave][r] = fmaf(w, E::load(cp + r), s_o[wave][r] * f);
    }
    if (lane == 0) s_m[wave] = m, s_l[wave] = l;
    __syncthreads();
    const float mx = fmaxf(fmaxf(s_m[0], s_m[1]), fmaxf(s_m[2], s_m[3]));
    const float sink = a.finish.sink ? a.finish.sink[head] : LA_NEG;
    float f[4], sum = expf(sink - mx);
#pragma unroll
    for (int w = 0; w < 4; ++w) f[w] = s_l[w] > 0.0f ? expf(s_m[w] - mx) : 0.0f, sum += s_l[w] * f[w];
    const float gate = head_gate<sizeof(T) == 4>(a.finish, row, head);
    for (int r = threadIdx.x; r < RO; r += 256)
        ((T *)a.out)[pr * a.ldq + r] = E::pack((s_o[0][r] * f[0] + s_o[1][r] * f[1] + s_o[2][r] * f[2] + s_o[3][r] * f[3]) * gate / sum);
}

template <class E, class X>
__global__ void __launch_bounds__(256) k_latent_append(const LatentAppend a) {
    __shared__ float red[4];
    latent_append_row<E, X, 256>(a, blockIdx.x, red);
}

// One workgroup per row: the query latent's norm, the latent's norm into the page, and the shared key part's rotation.
template <class E>
__global__ void __launch_bounds__(256) k_latent_prep(const LatentPrepArgs a) {
    typedef typename E::type T;
    __shared__ float red[2][4];
    const int m = blockIdx.x;
    if (a.cq) {
        const T *q = (const T *)a.raw + (size_t)m * a.ld;
        float ss = 0.0f;
        for (int i = threadIdx.x; i < a.Q; i += 256) ss = fmaf(E::load(q + i), E::load(q + i), ss);
        ss = lanes_sum(ss);
        if ((threadIdx.x & 63) == 0) red[0][threadIdx.x >> 6] = ss;
        __syncthreads();
        const float inv = 1.0f / sqrtf(((red[0][0] + red[0][1]) + (red[0][2] + red[0][3])) / (float)a.Q + a.eps);
        T *cq = (T *)a.cq + (size_t)m * a.ldc;
        for (int i = threadIdx.x; i < a.Q; i += 256) cq[i] = E::pack(E::load(q + i) * inv * (a.q_norm ? a.q_norm[i] : 1.0f));
    }
    if (a.own) latent_cache_row<E, 256>(a, m, red[1]);
}

template <class E>
__global__ void __launch_bounds__(256) k_rotate_heads(const RotateArgs a) {
    rotate_row<E, 256>(a, blockIdx.x);
}

}  // namespace

int latent_attn_tiles(int n_rows, int H) { return (n_rows * H + LA_PAIRS - 1) / LA_PAIRS; }

size_t latent_attn_ws_floats(int M, int H, int R, int splits) { return splits > 1 ? (size_t)splits * M * H * (((R + 7) & ~7) + 2) : 0; }

int latent_attn_launch(int dtype, const LatentAttnArgs &a, hipStream_t st) {
    if (a.M <= 0) return PIE_OK;
    PIE_REQUIRE(a.R > 0 && a.R <= LA_RMAX && a.H > 0 && a.H <= 65535, PIE_E_SHAPE, "latent attention: kv_rank must be 1 .. 2048");
    PIE_REQUIRE(a.splits >= 1 && (a.splits == 1 || a.ws), PIE_E_ARG, "latent attention: a key split needs its workspace");
    PIE_REQUIRE(a.ldq % 8 == 0 && a.ldr % 8 == 0 && a.R <= a.ldr && (a.ldq == a.ldr || (a.ldq < a.ldr && a.q_rot && a.ld_rot % 8 == 0)), PIE_E_ALIGN, "latent attention: row strides");
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
#define LA_GO(N) hipLaunchKernelGGL(k_latent_attn<N>, grid, dim3(256), 0, st, a)
    if (rc <= 2) LA_GO(2);
    else if (rc <= 4) LA_GO(4);
    else if (rc <= 6) LA_GO(6);
    else if (rc <= 8) LA_GO(8);
    else if (rc <= 10) LA_GO(10);
    else if (rc <= 12) LA_GO(12);
    else LA_GO(16);
#undef LA_GO
    PIE_LAUNCH_CHECK();
    if (a.splits > 1 && a.combine) {
        const LatentMerge m = {a.ws, a.splits, a.M, a.H, a.ldq, a.finish};
        hipLaunchKernelGGL(k_latent_combine, dim3((unsigned)(a.M * a.H)), dim3(128), 0, st, m, (u16 *)a.out);
        PIE_LAUNCH_CHECK();
    }
    return PIE_OK;
}

int latent_append_launch(int dtype, const LatentAppend &a, hipStream_t st) {
    if (a.M <= 0) return PIE_OK;
    const dim3 grid((unsigned)a.M);
    if (dtype == PIE_F32) hipLaunchKernelGGL((k_latent_append<ElemF32, ElemF32>), grid, dim3(256), 0, st, a);
    else if (a.raw16) hipLaunchKernelGGL((k_latent_append<ElemBF16, ElemBF16>), grid, dim3(256), 0, st, a);
    else hipLaunchKernelGGL((k_latent_append<ElemBF16, ElemF32>), grid, dim3(256), 0, st, a);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

int latent_prep_launch(int dtype, const LatentPrepArgs &a, hipStream_t st) {
    if (a.M <= 0) return PIE_OK;
    PIE_REQUIRE(a.rot.dims >= 0 && a.rot.dims <= a.T && a.rot.dims % 2 == 0 && (a.rot.dims == 0 || a.rot.freq), PIE_E_SHAPE, "latent attention: bad rotation");
    if (dtype == PIE_F32) hipLaunchKernelGGL(k_latent_prep<ElemF32>, dim3((unsigned)a.M), dim3(256), 0, st, a);
    else hipLaunchKernelGGL(k_latent_prep<ElemBF16>, dim3((unsigned)a.M), dim3(256), 0, st, a);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

int rotate_heads_launch(int dtype, const RotateArgs &a, hipStream_t st) {
    if (a.M <= 0 || a.rot.dims <= 0) return PIE_OK;
    PIE_REQUIRE(a.rot.dims % 2 == 0 && a.rot.dims <= a.stride && a.rot.freq, PIE_E_SHAPE, "rotation: an even number of a head's numbers");
    if (dtype == PIE_F32) hipLaunchKernelGGL(k_rotate_heads<ElemF32>, dim3((unsigned)a.M), dim3(256), 0, st, a);
    else hipLaunchKernelGGL(k_rotate_heads<ElemBF16>, dim3((unsigned)a.M), dim3(256), 0, st, a);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}
