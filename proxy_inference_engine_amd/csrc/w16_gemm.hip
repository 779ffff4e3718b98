// w16_gemm.hip -- nn.Linear with 16-bit weights on many rows: the launcher of k_w16l_gemm (w16_gemm.hpp), the repack into its W16M tiles, and the
// C entry points over both.  Part of libpie_base.so: the dense prompt path, the vision tower and the layer-stack models multiply through it.
#include <mutex>

#include "mfma_store.hpp"  // w4m_pack, the LDS-transposed output epilogue, k_w4l_reduce
#include "prefill_attn.hpp"  // MfmaT, f32x16_t

typedef __attribute__((address_space(3))) void w4l_lds_void;
#include "w16_gemm.hpp"

// y[m, n] = T(y[m, n] + b[n]), any N (two columns per thread; rows of odd length end in a single column)
template <class T>
__global__ void k_bias_any(u16 *y, const u16 *b, int M, int N) {
    const int n2 = (N + 1) >> 1;
    const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= (size_t)M * n2) return;
    const int m = (int)(i / n2), n = (int)(i % n2) * 2;
    u16 *p = y + (size_t)m * N + n;
    p[0] = T::from_f32(T::to_f32(p[0]) + T::to_f32(b[n]));
    if (n + 1 < N) p[1] = T::from_f32(T::to_f32(p[1]) + T::to_f32(b[n + 1]));
}

// y[m, :] = T(y[m, :] + bias) for any N (behind a K split, whose slabs are reduced before the bias)
int bias_any_launch(int dtype, void *y, const void *bias, int M, int N, hipStream_t st) {
    const size_t n = (size_t)M * ((N + 1) >> 1);
    const dim3 grid((unsigned)((n + 255) / 256)), block(256);
    if (dtype == PIE_BF16) hipLaunchKernelGGL(k_bias_any<BF16>, grid, block, 0, st, (u16 *)y, (const u16 *)bias, M, N);
    else hipLaunchKernelGGL(k_bias_any<F16>, grid, block, 0, st, (u16 *)y, (const u16 *)bias, M, N);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

// ---------------------------------------------------------------- 16-bit weights, many rows (w16_gemm.hpp)

static char *g_w16_zero = nullptr;  // 4 KiB of zeros: the weight tile of the ring's dummy steps
static std::mutex g_w16_mutex;
int w16_zero_block(const char **out) {
    std::lock_guard<std::mutex> lock(g_w16_mutex);
    if (!g_w16_zero) {
        PIE_HIP_TRY(hipMalloc((void **)&g_w16_zero, W16M_TILE_BYTES));
        PIE_HIP_TRY(hipMemset(g_w16_zero, 0, W16M_TILE_BYTES));
    }
    *out = g_w16_zero;
    return PIE_OK;
}

size_t w16m_size(int N, int K) { return w16m_bytes(N, K); }
// row-major [N][K] (any N, K) -> W16M
int w16m_from_rows_launch(const void *w, int N, int K, void *w16m, hipStream_t st) {
    const char *zero;
    if (const int rc = w16_zero_block(&zero)) return rc;  // (first use of the format: never under stream capture)
    const int groups = (K + 63) / 64;
    const size_t pieces = w16m_bytes(N, K) / 16;
    hipLaunchKernelGGL(k_rows_to_w16m, dim3((unsigned)((pieces + 255) / 256)), dim3(256), 0, st, (const u16 *)w, N, K, groups, pieces, (uint4 *)w16m);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}
// W16S units (the dense decode stream) -> W16M, packed row order
int w16m_from_w16s_launch(const void *w16s, int N, int K, void *w16m, hipStream_t st) {
    const char *zero;
    if (const int rc = w16_zero_block(&zero)) return rc;
    const int groups = (K + 63) / 64;
    const size_t pieces = w16m_bytes(N, K) / 16;
    hipLaunchKernelGGL(k_w16s_to_w16m, dim3((unsigned)((pieces + 255) / 256)), dim3(256), 0, st, (const uint4 *)w16s, N, K, (K + 511) / 512, groups, pieces,
                       (uint4 *)w16m);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

// Decomposition: row tile (64 / 128 / 256 rows), strips per wave (workgroup = 128 or 256 columns) and K split, by a small cost model
// calibrated on tools/w16_bench sweep (8B and vision-tower shapes, 64 .. 4096 rows): a K step of a (32 mb) x (128 sw) tile costs
// t(mb, sw) us -- larger tiles are cheaper per MFMA (0.125 us per 32 x 32 block pair for 64 x 128, 0.09 for 256 x 256) but quantise worse --
// less when part of the chip idles (the large tiles are power-bound: the clock rises); workgroups run in rounds of 256; few rows
// are bound by the weight stream (~5.5 TB/s); a launch costs ~4 us of ramp, prologue and epilogue; a K split writes and re-reads its fp32
// slabs and launches the reduce.
struct W16Plan {
    int mb, sw, S;
};
static int g_w16_plan_override[3] = {0, 0, 0};  // developer override (tools/w16_bench)
static int g_w16_block[2] = {4, 8};              // XCD-local traversal block (row tiles x column tiles)
#ifdef W16L_PROF
static unsigned long long *g_w16_prof = nullptr;
#endif
static int w16_even_splits(int groups, int S) {  // the largest split count <= S whose ceil-sized runs are all non-empty
    for (;;) {
        const int per = (groups + S - 1) / S, s2 = (groups + per - 1) / per;
        if (s2 == S) return S;
        S = s2;
    }
}
static W16Plan w16_plan(int M, int N, int K, bool no_split = false) {
    const int groups = (K + 63) / 64;
    if (g_w16_plan_override[0]) return {g_w16_plan_override[0], g_w16_plan_override[1], w16_even_splits(groups, g_w16_plan_override[2])};
    const int mb_max = M <= 64 ? 2 : (M <= 128 ? 4 : 8);
    W16Plan best = {mb_max, 2, 1};
    double best_us = 1e30;
    // t(mb, sw) = light + (full - light) * load: one partial round of workgroups runs at a higher clock than sustained full rounds
    static const double t_light[4][3] = {{0, 0, 0}, {0, 0.25, 0.42}, {0, 0.31, 0.60}, {0, 0.50, 1.45}};  // [log2 mb][sw]
    static const double t_rows[4][3] = {{0, 0, 0}, {0, 0.25, 0.45}, {0, 0.48, 0.80}, {0, 0.83, 1.45}};
    static const double t_tall[4][3] = {{0, 0, 0}, {0, 0.31, 0.53}, {0, 0.46, 0.84}, {0, 0.90, 1.45}};  // many row tiles: small tiles re-read the weights from beyond their XCD's L2
    const double (&t_full)[4][3] = M > 512 ? t_tall : t_rows;
    const double stream_us = 2.0 * N * (64.0 * groups) / 5.5e6;
    for (int S = 1; S <= (no_split ? 1 : 16) && (S == 1 || 8 * S <= groups); ++S)
        for (int mb = mb_max; mb >= 2; mb >>= 1)
            for (int sw = 2; sw >= (no_split ? 2 : 1); --sw) {
                const int wgs = ((N + 128 * sw - 1) / (128 * sw)) * ((M + 32 * mb - 1) / (32 * mb)) * S;
                const int steps = ((groups + S - 1) / S + 3) & ~3;
                const int rounds = (wgs + 255) / 256;
                const double load = rounds > 1 ? 1.0 : (double)wgs / 256.0;
                const int mi = mb == 8 ? 3 : (mb == 4 ? 2 : 1);
                double us = rounds * steps * (t_light[mi][sw] + (t_full[mi][sw] - t_light[mi][sw]) * load);
                us = (us > stream_us ? us : stream_us) + 4.0;
                if (S > 1) us += (double)M * N * 4.0 * (2 * S + 0.5) / 4.0e6 + 2.0;
                if (us < best_us) best_us = us, best = {mb, sw, S};
            }
    best.S = w16_even_splits(groups, best.S);
    return best;
}
int w16l_splits(int M, int N, int K) { return w16_plan(M, N, K).S; }
size_t w16l_workspace_bytes(int M, int N, int K) {
    if (N & 3) return 0;
    const int s = w16l_splits(M, N, K);
    return s > 1 ? (size_t)s * M * N * sizeof(float) : 0;
}

// y [M, N] = x . W^T (+ bias), W in W16M tiles of an [N, K] Linear; x: M rows of ldx elements (0 = packed) holding 64 ceil(K / 64) used
// columns, zeros past K.
// swiglu_act (nullable): the packed gate|up matrix and the caller wants the MLP activation [M, N / 2] there; *fused says whether it got it.
// workspace: w16l_workspace_bytes() of device scratch (may be null when that is 0).
// ldy: row stride of the output that is written (y, or the activation; 0 = packed), a multiple of 4.
int w16l_gemm_launch(int dtype, const void *w16m, const void *x, int ldx, int M, int N, int K, void *y, void *workspace, hipStream_t st, const void *bias,
                     void *swiglu_act, bool *fused, int ldy) {
    if (fused) *fused = false;
    const int Kx = 64 * ((K + 63) / 64);
    if (ldx == 0) ldx = Kx;
    PIE_REQUIRE(ldx >= Kx && ldx % 8 == 0 && (size_t)256 * ldx * 2 < (1ull << 32), PIE_E_SHAPE,
                "16-bit GEMM: x rows must hold 64 * ceil(K / 64) elements (zeros past K) at a stride that is a multiple of 8");
    PIE_REQUIRE(M >= 1 && N > 0 && K > 0, PIE_E_SHAPE, "16-bit GEMM: empty operand");
    PIE_REQUIRE(pie_aligned(w16m, 16) && pie_aligned(x, 16) && pie_aligned(y, 8) && (!bias || pie_aligned(bias, (N & 3) ? 2 : 8)), PIE_E_ALIGN, "16-bit GEMM: 16-byte alignment required");
    PIE_REQUIRE(dtype == PIE_BF16 || dtype == PIE_F16, PIE_E_ARG, "16-bit GEMM: dtype must be PIE_BF16 or PIE_F16");
    // swiglu_act without `fused`: the caller has no fallback (the C ABI's fused MLP): plan without a K split, two strips per wave
    W16Plan plan = w16_plan(M, N, K, (swiglu_act && !fused) || (N & 3));  // (the fp32 slabs of a K split are written 16 bytes at a time)
    const bool sg = swiglu_act && plan.S == 1;
    if (sg) plan.sw = 2;  // (the fused activation is built for two strips per wave)
    PIE_REQUIRE(plan.S == 1 || workspace, PIE_E_ARG, "16-bit GEMM: this shape splits K and needs its workspace");
    W16Args a = {};
    int rc = w16_zero_block(&a.zero);
    if (rc) return rc;
    PIE_REQUIRE(!sg || N % 8 == 0, PIE_E_SHAPE, "16-bit GEMM: a fused SwiGLU needs N % 8 == 0");
    const int out_cols = sg ? N / 2 : N;
    if (ldy == 0 || (swiglu_act && !sg)) ldy = out_cols;  // (a declined fusion writes the packed y)
    PIE_REQUIRE(ldy >= out_cols, PIE_E_SHAPE, "16-bit GEMM: output row stride must cover the row");
    PIE_REQUIRE(plan.S == 1 || ldy == N, PIE_E_SHAPE, "16-bit GEMM: a K-split shape writes packed rows");
    a.w16m = (const char *)w16m, a.x = (const u16 *)x, a.M = M, a.N = N, a.K = Kx, a.ldx = ldx, a.ldy = ldy;
    a.y = (u16 *)(sg ? swiglu_act : y), a.part = plan.S > 1 ? (float *)workspace : nullptr;
    a.bias = plan.S > 1 ? nullptr : (const u16 *)bias;
    a.tm = (M + 32 * plan.mb - 1) / (32 * plan.mb), a.tn = (N + 128 * plan.sw - 1) / (128 * plan.sw);
    a.bm = g_w16_block[0] < a.tm ? g_w16_block[0] : a.tm, a.bc = g_w16_block[1];
#ifdef W16L_PROF
    a.prof = g_w16_prof;
#endif
    a.narrow = a.tn < 8 && a.tm >= 8;
    const dim3 grid((unsigned)(a.narrow ? 8 * ((a.tm + 7) / 8) * a.tn : 8 * ((a.tn + 7) / 8) * a.tm), (unsigned)plan.S);
#define W16_GO(TT, MB_, SW_, SG_) hipLaunchKernelGGL((k_w16l_gemm<TT, MB_, SW_, SG_>), grid, dim3(256), 0, st, a)
#define W16_SW(TT, MB_) \
    if (sg) W16_GO(TT, MB_, 2, true); \
    else if (plan.sw == 2) W16_GO(TT, MB_, 2, false); \
    else W16_GO(TT, MB_, 1, false)
#define W16_MB(TT) \
    if (plan.mb == 2) { W16_SW(TT, 2); } \
    else if (plan.mb == 4) { W16_SW(TT, 4); } \
    else { W16_SW(TT, 8); }
    if (dtype == PIE_BF16) { W16_MB(BF16) } else { W16_MB(F16) }
#undef W16_MB
#undef W16_SW
#undef W16_GO
    PIE_LAUNCH_CHECK();
    if (sg && fused) *fused = true;
    if (plan.S > 1) {
        const size_t MN = (size_t)M * N;
        const dim3 rg((unsigned)((MN / 4 + 255) / 256));
        if (dtype == PIE_BF16) hipLaunchKernelGGL(k_w4l_reduce<BF16>, rg, dim3(256), 0, st, a.part, plan.S, MN, (u16 *)y);
        else hipLaunchKernelGGL(k_w4l_reduce<F16>, rg, dim3(256), 0, st, a.part, plan.S, MN, (u16 *)y);
        PIE_LAUNCH_CHECK();
        if (bias) return bias_any_launch(dtype, y, bias, M, N, st);
    }
    return PIE_OK;
}

extern "C" {

size_t pie_w16m_bytes(int N, int K) { return N > 0 && K > 0 ? w16m_size(N, K) : 0; }

int pie_repack_w16m(const void *w, int N, int K, int dtype, void *w16m, void *stream) {
    PIE_REQUIRE(w && w16m, PIE_E_ARG, "pie_repack_w16m: null pointer");
    PIE_REQUIRE(N > 0 && K > 0, PIE_E_SHAPE, "pie_repack_w16m: empty matrix");
    PIE_REQUIRE(dtype == PIE_BF16 || dtype == PIE_F16, PIE_E_ARG, "pie_repack_w16m: dtype must be PIE_BF16 or PIE_F16");
    PIE_REQUIRE(pie_aligned(w, 16) && pie_aligned(w16m, 256), PIE_E_ALIGN, "pie_repack_w16m: w needs 16-byte, w16m 256-byte alignment");
    return w16m_from_rows_launch(w, N, K, w16m, (hipStream_t)stream);
}

size_t pie_linear_w16m_workspace(int M, int N, int K) { return M > 0 && N > 0 && K > 0 ? w16l_workspace_bytes(M, N, K) : 0; }

int pie_linear_w16m(const void *x, int ldx, const void *w16m, const void *bias, int M, int N, int K, int dtype, void *y, int ldy, int swiglu,
                    void *workspace, size_t workspace_bytes, void *stream) {
    PIE_REQUIRE(x && w16m && y, PIE_E_ARG, "pie_linear_w16m: null pointer");
    PIE_REQUIRE(M > 0 && N > 0 && K > 0, PIE_E_SHAPE, "pie_linear_w16m: empty operand");
    PIE_REQUIRE(!swiglu || N % 8 == 0, PIE_E_SHAPE, "pie_linear_w16m: the fused SiLU * up needs N % 8 == 0");
    PIE_REQUIRE(dtype == PIE_BF16 || dtype == PIE_F16, PIE_E_ARG, "pie_linear_w16m: dtype must be PIE_BF16 or PIE_F16");
    PIE_REQUIRE(pie_aligned(x, 16) && pie_aligned(w16m, 16) && pie_aligned(y, 16) && (!bias || pie_aligned(bias, (N & 3) ? 2 : 8)), PIE_E_ALIGN,
                "pie_linear_w16m: 16-byte alignment required");
    const size_t need = swiglu ? 0 : w16l_workspace_bytes(M, N, K);
    PIE_REQUIRE(need == 0 || (workspace && workspace_bytes >= need), PIE_E_ARG, "pie_linear_w16m: workspace smaller than pie_linear_w16m_workspace(M, N, K)");
    return w16l_gemm_launch(dtype, w16m, x, ldx, M, N, K, swiglu ? nullptr : y, workspace, (hipStream_t)stream, bias, swiglu ? y : nullptr, nullptr, ldy);
}

}  // extern "C"
