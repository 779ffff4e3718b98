// window_attn.hip -- attention of long portions with keys and values spelled out: flash attention on the matrix cores, one key and one value vector per
// head and token, causal, with an optional sliding window.
//
// For a decoded token the latent form (latent_attn.hip) reads the least; for a prompt it would multiply R numbers per score where the head's own key
// has only `dim`.  So a run of many rows first copies the latents it can see out of the pages, multiplies them into all heads' keys and values (one
// GEMM), and attends here.
//
// A workgroup owns 128 query rows (4 waves x 32) of one head and walks the 32-key blocks of their union of windows; K and V blocks are staged once in
// LDS.  Per wave and block: S^T = K . Q^T (32x32x16 MFMAs, keys in registers, rows in lanes), online softmax in fp32, O^T += V^T . P^T with V read
// transposed from LDS and P split into hi + lo bf16 halves.  Keys and queries may have a second part (a rotated one; the keys' is the same for all heads and comes
// from the latents' rows): scores simply run over both.  Blocks outside a wave's own window are skipped, blocks inside it for every row are not masked.
#include "mfma_store.hpp"  // w4m_pack
#include "prefill_attn.hpp"
#include "stack_types.hpp"

namespace {

// the run a long-run tile or context row belongs to, and what precedes it
__device__ __forceinline__ int wa_first(const RowRun &r, int window) { return window > 0 ? max(0, r.pos0 - window + 1) : 0; }

__global__ void __launch_bounds__(64) k_latent_gather(const RowRun *runs, int n_runs, int window, const int *table, int table_width, int n_seqs, int n_pages, const u16 *slab,
                                                      int ldr, u16 *out, int ld_out) {
    int i = blockIdx.x, r = 0;
    for (;;) {
        const int n = runs[r].pos0 + runs[r].n_rows - wa_first(runs[r], window);
        if (i < n || r + 1 >= n_runs) break;
        i -= n, ++r;
    }
    const int t = wa_first(runs[r], window) + i;
    const int page = (int)min((unsigned)table[(size_t)min(runs[r].seq, n_seqs - 1) * table_width + min(t / PAGE_TOKENS, table_width - 1)], (unsigned)n_pages - 1u);
    const u16 *src = slab + ((size_t)page * PAGE_TOKENS + (t & (PAGE_TOKENS - 1))) * ldr;
    for (int c = threadIdx.x * 8; c < ldr; c += 512) *(uint4 *)(out + (size_t)blockIdx.x * ld_out + c) = *(const uint4 *)(src + c);
}

template <int DK, int DV>  // scores over up to DK numbers, values of up to DV
__global__ void __launch_bounds__(256, DV <= 128 ? 2 : 1) k_window_attn(const WindowAttnArgs a) {
    constexpr int KC = DK / 8, VC = DV / 8, KS = DK / 16, DT = DV / 32, KPT = (32 * KC + 255) / 256, VPT = (32 * VC + 255) / 256;
    __shared__ __attribute__((aligned(16))) char k_lds[32 * 2 * DK], v_lds[32 * 2 * DV];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int c = lane & 31, h = lane >> 5;
    const int head = (int)blockIdx.x % a.H;  // fastest: an XCD keeps meeting the same heads' keys
    int tile = (int)gridDim.x / a.H - 1 - (int)blockIdx.x / a.H, r = 0;  // later rows (more keys) first
    int ctx = 0;
    for (;;) {
        const int n = (a.runs[r].n_rows + 127) / 128;
        if (tile < n || r + 1 >= a.n_runs) break;
        ctx += a.runs[r].pos0 + a.runs[r].n_rows - wa_first(a.runs[r], a.window);
        tile -= n, ++r;
    }
    const RowRun run = a.runs[r];
    const int w0 = tile * 128;                    // first row of the workgroup inside the run
    if (w0 >= run.n_rows) return;
    const int first = wa_first(run, a.window);    // position of the run's context row 0
    const int t_last = run.pos0 + min(w0 + 127, run.n_rows - 1);
    const int t_first = a.window > 0 ? max(0, run.pos0 + w0 - a.window + 1) : 0;
    const u16 *kbase = a.kv + (size_t)ctx * a.ld_kv + head * a.D8, *vbase = a.kv + (size_t)ctx * a.ld_kv + a.H * a.D8 + head * a.V8;

    const u16 *krot = a.k_rot + (size_t)ctx * a.ld_krot;
    uint4 kr[KPT], vr[VPT];
    auto fetch = [&](int t0) {
#pragma unroll
        for (int i = 0; i < KPT; ++i) {
            const int x = threadIdx.x + 256 * i, row = x / KC, d = 8 * (x % KC);
            const int t = min(max(t0 + row, first), t_last);  // (clamped rows are masked)
            const bool in = 32 * KC >= 256 || x < 32 * KC;
            const u16 *p = d < a.D8 ? kbase + (size_t)(t - first) * a.ld_kv + d : krot + (size_t)(t - first) * a.ld_krot + d - a.D8;
            kr[i] = in && d < a.D8 + a.T8 ? *(const uint4 *)p : make_uint4(0, 0, 0, 0);
        }
#pragma unroll
        for (int i = 0; i < VPT; ++i) {
            const int x = threadIdx.x + 256 * i, row = x / VC, d = 8 * (x % VC);
            const int t = min(max(t0 + row, first), t_last);
            const bool in = 32 * VC >= 256 || x < 32 * VC;
            vr[i] = in && d < a.V8 ? *(const uint4 *)(vbase + (size_t)(t - first) * a.ld_kv + d) : make_uint4(0, 0, 0, 0);
        }
    };
    const int b0 = t_first / 32, b1 = t_last / 32;
    fetch(b0 * 32);

    const int r0 = w0 + 32 * wave;                // the wave's first row
    const bool busy = r0 < run.n_rows;
    const int row = run.row0 + min(r0 + c, run.n_rows - 1);
    const int t_q = run.pos0 + min(r0 + c, run.n_rows - 1), t_min = a.window > 0 ? t_q - a.window + 1 : 0;
    const int q_lo = run.pos0 + r0, q_hi = run.pos0 + min(r0 + 31, run.n_rows - 1);  // the wave's positions
    const int k_lo = a.window > 0 ? q_lo - a.window + 1 : 0, k_full = a.window > 0 ? q_hi - a.window + 1 : 0;
    uint4 qf[KS];
#pragma unroll
    for (int s = 0; s < KS; ++s) {
        const int d = 16 * s + 8 * h;
        const u16 *p = d < a.D8 ? a.q + (size_t)row * a.ld_q + head * a.D8 + d : a.q_rot + (size_t)row * a.ld_q + head * a.T8 + d - a.D8;
        qf[s] = d < a.D8 + a.T8 ? *(const uint4 *)p : make_uint4(0, 0, 0, 0);
    }
    const float sl2 = a.scale * ATTN_LOG2E;
    f32x16_t oacc[DT];
#pragma unroll
    for (int d = 0; d < DT; ++d)
#pragma unroll
        for (int i = 0; i < 16; ++i) oacc[d][i] = 0.0f;
    float m_run = ATTN_NEG, l_run = 0.0f;
    const int grp = lane >> 4, tq = (lane & 15) >> 2, tp = lane & 3;

    for (int b = b0; b <= b1; ++b) {
        const int t0 = b * 32;
        __syncthreads();
#pragma unroll
        for (int i = 0; i < KPT; ++i) {
            const int x = threadIdx.x + 256 * i;
            if (32 * KC >= 256 || x < 32 * KC) *(uint4 *)(k_lds + pa_off<DK>(x / KC, x % KC)) = kr[i];
        }
#pragma unroll
        for (int i = 0; i < VPT; ++i) {
            const int x = threadIdx.x + 256 * i;
            if (32 * VC >= 256 || x < 32 * VC) *(uint4 *)(v_lds + pa_off<DV>(x / VC, x % VC)) = vr[i];
        }
        __syncthreads();
        if (b < b1) fetch(t0 + 32);
        if (!busy || t0 > q_hi || t0 + 31 < k_lo) continue;
        f32x16_t sacc;
#pragma unroll
        for (int i = 0; i < 16; ++i) sacc[i] = 0.0f;
#pragma unroll
        for (int s = 0; s < KS; ++s) sacc = MfmaT<BF16>::run(*(const uint4 *)(k_lds + pa_off<DK>(c, 2 * s + h)), qf[s], sacc);
        // register i <-> key t0 + (i & 3) + 8 (i >> 2) + 4 h
        float sc[16], mloc = ATTN_NEG;
        if (t0 + 31 <= q_lo && t0 >= k_full) {  // wave-uniform: every row of the wave sees the whole block
#pragma unroll
            for (int i = 0; i < 16; ++i) sc[i] = sacc[i] * sl2, mloc = fmaxf(mloc, sc[i]);
        } else {
#pragma unroll
            for (int i = 0; i < 16; ++i) {
                const int t = t0 + (i & 3) + 8 * (i >> 2) + 4 * h;
                sc[i] = t <= t_q && t >= t_min ? sacc[i] * sl2 : ATTN_NEG;
                mloc = fmaxf(mloc, sc[i]);
            }
        }
        mloc = xor32_max(mloc);
        if (mloc > m_run) {
            const float alpha = attn_exp2(m_run - mloc);
            l_run *= alpha;
#pragma unroll
            for (int d = 0; d < DT; ++d)
#pragma unroll
                for (int i = 0; i < 16; ++i) oacc[d][i] *= alpha;
            m_run = mloc;
        }
        u32 phi[8], plo[8];
#pragma unroll
        for (int i = 0; i < 16; i += 2) {
            const float pa = sc[i] > ATTN_NEG ? attn_exp2(sc[i] - m_run) : 0.0f, pb = sc[i + 1] > ATTN_NEG ? attn_exp2(sc[i + 1] - m_run) : 0.0f;
            l_run += pa + pb;
            const u32 hi = w4m_pack<BF16>(pa, pb);
            phi[i >> 1] = hi;
            plo[i >> 1] = w4m_pack<BF16>(pa - lo_f32<BF16>(hi), pb - hi_f32<BF16>(hi));
        }
#pragma unroll
        for (int s = 0; s < 2; ++s) {
            const uint4 bh = make_uint4(phi[4 * s], phi[4 * s + 1], phi[4 * s + 2], phi[4 * s + 3]);
            const uint4 bl = make_uint4(plo[4 * s], plo[4 * s + 1], plo[4 * s + 2], plo[4 * s + 3]);
#pragma unroll
            for (int d = 0; d < DT; ++d) {
                const int ch = 4 * d + 2 * (grp & 1) + (tp >> 1);
                const v4i16_t lo4 = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
                    (__attribute__((address_space(3))) v4i16_t *)(v_lds + pa_off<DV>(16 * s + 4 * h + tq, ch) + 8 * (tp & 1)));
                const v4i16_t hi4 = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
                    (__attribute__((address_space(3))) v4i16_t *)(v_lds + pa_off<DV>(16 * s + 8 + 4 * h + tq, ch) + 8 * (tp & 1)));
                const uint2 a0 = __builtin_bit_cast(uint2, lo4), a1 = __builtin_bit_cast(uint2, hi4);
                const uint4 vf = make_uint4(a0.x, a0.y, a1.x, a1.y);
                oacc[d] = MfmaT<BF16>::run(vf, bh, oacc[d]);
                oacc[d] = MfmaT<BF16>::run(vf, bl, oacc[d]);
            }
        }
    }
    const float l = xor32_sum(l_run);
    if (r0 + c >= run.n_rows) return;
    const float inv = head_gate<false>(a.finish, row, head) / (l + head_sink2(a.finish, head, m_run));
    u16 *dst = a.out + (size_t)row * a.ld_out + head * a.V8;
#pragma unroll
    for (int d = 0; d < DT; ++d)
#pragma unroll
        for (int k = 0; k < 4; ++k)  // registers 4k .. 4k + 3 <-> dims 32 d + 8 k + 4 h + {0..3}
            if (32 * d + 8 * k + 4 * h < a.V8)
                *(uint2 *)(dst + 32 * d + 8 * k + 4 * h) = make_uint2(w4m_pack<BF16>(oacc[d][4 * k] * inv, oacc[d][4 * k + 1] * inv),
                                                                      w4m_pack<BF16>(oacc[d][4 * k + 2] * inv, oacc[d][4 * k + 3] * inv));
}

}  // namespace

int latent_gather_launch(const RowRun *runs, int n_runs, int n_ctx, int window, const int *table, int table_width, int n_seqs, int n_pages, const void *slab, int ldr,
                         void *out, int ld_out, hipStream_t st) {
    hipLaunchKernelGGL(k_latent_gather, dim3((unsigned)n_ctx), dim3(64), 0, st, runs, n_runs, window, table, table_width, n_seqs, n_pages, (const u16 *)slab, ldr, (u16 *)out, ld_out);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

int window_attn_launch(const WindowAttnArgs &a, int n_tiles, hipStream_t st) {
    const int k = a.D8 + a.T8, v = a.V8;
    PIE_REQUIRE(k <= WINDOW_ATTN_MAX_DIM && v <= WINDOW_ATTN_MAX_DIM && (a.T8 == 0 || (a.q_rot && a.k_rot && a.ld_krot % 8 == 0)), PIE_E_SHAPE, "window attention: heads of at most 256 numbers");
    const dim3 grid((unsigned)(n_tiles * a.H));
#define WA_GO(K_, V_) hipLaunchKernelGGL((k_window_attn<K_, V_>), grid, dim3(256), 0, st, a)
    if (k <= 32 && v <= 32) WA_GO(32, 32);
    else if (k <= 64 && v <= 64) WA_GO(64, 64);
    else if (k <= 128 && v <= 64) WA_GO(128, 64);
    else if (k <= 128 && v <= 128) WA_GO(128, 128);
    else if (k <= 192 && v <= 128) WA_GO(192, 128);
    else WA_GO(256, 256);
#undef WA_GO
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}
