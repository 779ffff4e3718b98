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
__device__ __forceinline__ int la_off(int row, int ch) {  // byte offset of 16-byte chunk ch of key row: XOR-swizzled, conflict-free for both kinds of reads
    const int sw = ((row & 3) << 2) | ((row >> 2) & 3);
    return row * (RC * 128) + 16 * (ch ^ (RC % 2 ? sw & 7 : sw));
}

template <int RC>  // latents of up to 64 RC numbers
__global__ void __launch_bounds__(256) k_latent_attn(const LatentAttnArgs a) {
    __shared__ __attribute__((aligned(16))) char s_c[LA_BK * RC * 128];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int c = lane & 15, g = lane >> 4;
    int run_i = 0, pair0 = blockIdx.x;
    if (a.single) {
        const int per_run = (a.H + 63) / 64;
        run_i = pair0 / per_run, pair0 %= per_run;
    } else {
        for (;;) {
            const int n = (a.runs[run_i].n_rows * a.H + 63) / 64;
            if (pair0 < n || run_i + 1 >= a.n_runs) break;
            pair0 -= n, ++run_i;
        }
    }
    pair0 *= 64;
    const RowRun tile = a.runs[run_i];
    const int last = min(64, tile.n_rows * a.H - pair0) - 1;
    if (last < 0) return;  // (a grid larger than the runs need)
    const int row_a = tile.row0 + pair0 / a.H, row_b = tile.row0 + (pair0 + last) / a.H;
    const int t_hi = a.pos[row_b], t_lo = a.window > 0 ? max(0, a.pos[row_a] - a.window + 1) : 0;
    const int nb = t_hi / LA_BK - t_lo / LA_BK + 1, per = (nb + a.splits - 1) / a.splits;
    const int b_begin = t_lo / LA_BK + (int)blockIdx.y * per, b_end = min(t_hi / LA_BK + 1, b_begin + per);

    const bool busy = 16 * wave <= last;
    const int p = pair0 + min(16 * wave + c, last);
    const int row = tile.row0 + p / a.H, head = p % a.H;
    const size_t pr = (size_t)row * a.H + head;
    const int t_q = a.pos[row], t_min = a.window > 0 ? t_q - a.window + 1 : 0;
    const u16 *qp = (const u16 *)a.q + pr * a.ldr;
    uint4 qf[2 * RC];
#pragma unroll
    for (int s = 0; s < 2 * RC; ++s) qf[s] = 32 * s + 8 * g < a.ldr ? *(const uint4 *)(qp + 32 * s + 8 * g) : make_uint4(0, 0, 0, 0);

    uint4 nx[RC];
    auto fetch = [&](int b) {
        const u16 *src = (const u16 *)a.slab + ((size_t)la_page(a, tile.seq, b * LA_BK) * PAGE_TOKENS + (b & 1) * LA_BK) * a.ldr;
#pragma unroll
        for (int i = 0; i < RC; ++i) {
            const int x = threadIdx.x + 256 * i, r = x / (8 * RC), ch = x % (8 * RC);
            nx[i] = 8 * ch < a.ldr ? *(const uint4 *)(src + (size_t)r * a.ldr + 8 * ch) : make_uint4(0, 0, 0, 0);
        }
    };
    la_f32x4 o[4 * RC];
#pragma unroll
    for (int r = 0; r < 4 * RC; ++r) o[r] = (la_f32x4){0.0f, 0.0f, 0.0f, 0.0f};
    float m_run = LA_NEG, l_run = 0.0f;
    const float sl2 = a.scale * LA_LOG2E;
    const int tq = (lane & 15) >> 2, tp = lane & 3;

    if (b_begin < b_end) fetch(b_begin);
    for (int b = b_begin; b < b_end; ++b) {
        __syncthreads();
#pragma unroll
        for (int i = 0; i < RC; ++i) {
            const int x = threadIdx.x + 256 * i;
            *(uint4 *)(s_c + la_off<RC>(x / (8 * RC), x % (8 * RC))) = nx[i];
        }
        __syncthreads();
        if (b + 1 < b_end) fetch(b + 1);
        if (!busy) continue;
        la_f32x4 s0 = {0.0f, 0.0f, 0.0f, 0.0f}, s1 = s0;
#pragma unroll
        for (int s = 0; s < 2 * RC; ++s) {
            const la_bf16x8 q = __builtin_bit_cast(la_bf16x8, qf[s]);
            const uint4 ka = *(const uint4 *)(s_c + la_off<RC>(c, 4 * s + g)), kb = *(const uint4 *)(s_c + la_off<RC>(16 + c, 4 * s + g));
            s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(la_bf16x8, ka), q, s0, 0, 0, 0);
            s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(la_bf16x8, kb), q, s1, 0, 0, 0);
        }
        // register i of s0 / s1 <-> key 32 b + 4 g + i (+ 16)
        const int t0 = b * LA_BK + 4 * g;
        float sc[8], mloc = LA_NEG;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const int t = t0 + (i & 3) + 16 * (i >> 2);
            sc[i] = (t <= t_q && t >= t_min) ? (i < 4 ? s0[i & 3] : s1[i & 3]) * sl2 : LA_NEG;
            mloc = fmaxf(mloc, sc[i]);
        }
        mloc = xor32_max(xor16_max(mloc));
        if (mloc > m_run) {
            const float alpha = exp2f(m_run - mloc);
            l_run *= alpha;
#pragma unroll
            for (int r = 0; r < 4 * RC; ++r) o[r] *= alpha;
            m_run = mloc;
        }
        u32 hi[4], lo[4];
#pragma unroll
        for (int i = 0; i < 8; i += 2) {
            const float pa = sc[i] > LA_NEG ? exp2f(sc[i] - m_run) : 0.0f, pb = sc[i + 1] > LA_NEG ? exp2f(sc[i + 1] - m_run) : 0.0f;
            l_run += pa + pb;
            const float ha = round_T<BF16>(pa), hb = round_T<BF16>(pb);
            hi[i >> 1] = pack2<BF16>(ha, hb);
            lo[i >> 1] = pack2<BF16>(pa - ha, pb - hb);
        }
        const la_bf16x8 ph = __builtin_bit_cast(la_bf16x8, make_uint4(hi[0], hi[1], hi[2], hi[3]));
        const la_bf16x8 pl = __builtin_bit_cast(la_bf16x8, make_uint4(lo[0], lo[1], lo[2], lo[3]));
#pragma unroll
        for (int r = 0; r < 4 * RC; ++r) {
            const int ch = 2 * r + (tp >> 1);
            const v4s_t a0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) v4s_t *)(s_c + la_off<RC>(4 * g + tq, ch) + 8 * (tp & 1)));
            const v4s_t a1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) v4s_t *)(s_c + la_off<RC>(16 + 4 * g + tq, ch) + 8 * (tp & 1)));
            const uint2 u0 = __builtin_bit_cast(uint2, a0), u1 = __builtin_bit_cast(uint2, a1);
            const la_bf16x8 ct = __builtin_bit_cast(la_bf16x8, make_uint4(u0.x, u0.y, u1.x, u1.y));
            o[r] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ct, ph, o[r], 0, 0, 0);
            o[r] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ct, pl, o[r], 0, 0, 0);
        }
    }
    const float l = xor32_sum(xor16_sum(l_run));
    if (16 * wave + c > last) return;
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

// merges the key splits of one (token, head) pair
__global__ void __launch_bounds__(128) k_latent_combine(const LatentAttnArgs a) {
    const size_t pr = blockIdx.x, MH = (size_t)a.M * a.H;
    const float *ml = a.ws + (size_t)a.splits * MH * a.ldr + pr * 2;
    float m = LA_NEG;
    for (int s = 0; s < a.splits; ++s)
        if (ml[s * MH * 2 + 1] > 0.0f) m = fmaxf(m, ml[s * MH * 2]);
    float l = 0.0f;
    for (int s = 0; s < a.splits; ++s) l += ml[s * MH * 2 + 1] > 0.0f ? ml[s * MH * 2 + 1] * exp2f(ml[s * MH * 2] - m) : 0.0f;
    const float inv = 1.0f / l;
    for (int r = threadIdx.x * 4; r < a.ldr; r += 512) {
        la_f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
        for (int s = 0; s < a.splits; ++s) {
            if (!(ml[s * MH * 2 + 1] > 0.0f)) continue;  // an empty split wrote no sums
            const float f = exp2f(ml[s * MH * 2] - m);
            const la_f32x4 v = *(const la_f32x4 *)(a.ws + (s * MH + pr) * a.ldr + r);
#pragma unroll
            for (int i = 0; i < 4; ++i) acc[i] = fmaf(f, v[i], acc[i]);
        }
        *(uint2 *)((u16 *)a.out + pr * a.ldr + r) = make_uint2(pack2<BF16>(acc[0] * inv, acc[1] * inv), pack2<BF16>(acc[2] * inv, acc[3] * inv));
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
#define LA_GO(N) hipLaunchKernelGGL(k_latent_attn<N>, grid, dim3(256), 0, st, a)
    if (rc <= 1) LA_GO(1);
    else if (rc <= 2) LA_GO(2);
    else if (rc <= 3) LA_GO(3);
    else if (rc <= 4) LA_GO(4);
    else if (rc <= 6) LA_GO(6);
    else if (rc <= 8) LA_GO(8);
    else if (rc <= 10) LA_GO(10);
    else LA_GO(16);
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
