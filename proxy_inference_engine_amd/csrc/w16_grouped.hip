// w16_grouped.hip -- forms of k_w16l_gemm (w16_gemm.hpp) that the layer-stack models add: epilogues with an activation, and the grouped product of a
// mixture's experts (every expert its own matrix and its own rows).
#include "mfma_store.hpp"
#include "prefill_attn.hpp"

typedef __attribute__((address_space(3))) void w4l_lds_void;
#include "w16_gemm.hpp"

int w16_zero_block(const char **out);  // w16_gemm.hip

static int w16_fill(W16Args &a, const void *w16m, const void *x, int ldx, int N, int K, void *y, int ldy) {
    const int Kx = 64 * ((K + 63) / 64);
    PIE_REQUIRE(N > 0 && K > 0, PIE_E_SHAPE, "16-bit GEMM: empty matrix");
    PIE_REQUIRE(ldx >= Kx && ldx % 8 == 0 && pie_aligned(w16m, 16) && pie_aligned(x, 16) && pie_aligned(y, 8), PIE_E_ALIGN, "16-bit GEMM: bad operand stride or alignment");
    if (int rc = w16_zero_block(&a.zero)) return rc;
    a.w16m = (const char *)w16m, a.x = (const u16 *)x, a.N = N, a.K = Kx, a.ldx = ldx, a.y = (u16 *)y, a.ldy = ldy;
    a.tn = (N + 255) / 256, a.bm = 4, a.bc = 8;
    return PIE_OK;
}

// y = T(act(x . W^T)), bf16; act: MFMA_ACT_NONE, MFMA_ACT_RELU2, MFMA_ACT_XIELU (alpha, beta: its factors) or MFMA_ACT_GELU of the interleaved matrix, N / 2 wide (bias bf16 [N], nullable)
int w16l_act_launch(const void *w16m, const void *x, int ldx, int M, int N, int K, void *y, int ldy, int act, float alpha, float beta, const void *bias, hipStream_t st) {
    W16Args a = {};
    if (int rc = w16_fill(a, w16m, x, ldx, N, K, y, ldy)) return rc;
    PIE_REQUIRE((size_t)256 * ldx * 2 < (1ull << 32), PIE_E_SHAPE, "16-bit GEMM: row stride too long");
    PIE_REQUIRE(act == MFMA_ACT_NONE || act == MFMA_ACT_RELU2 || act == MFMA_ACT_XIELU || (act == MFMA_ACT_GELU && N % 8 == 0), PIE_E_ARG, "16-bit GEMM: unknown activation");
    PIE_REQUIRE(!bias || (act == MFMA_ACT_GELU && pie_aligned(bias, 8)), PIE_E_ARG, "16-bit GEMM: a bias goes with the paired gelu");
    a.bias = (const u16 *)bias;
    int mb = 8;  // the largest row tile that still gives the chip a round of workgroups
    while (mb > 2 && (M <= 16 * mb || a.tn * ((M + 32 * mb - 1) / (32 * mb)) < 200)) mb >>= 1;
    a.M = M, a.tm = (M + 32 * mb - 1) / (32 * mb), a.bm = a.bm < a.tm ? a.bm : a.tm, a.act_alpha = alpha, a.act_limit = beta;
    a.narrow = a.tn < 8 && a.tm >= 8;
    const dim3 grid((unsigned)(a.narrow ? 8 * ((a.tm + 7) / 8) * a.tn : 8 * ((a.tn + 7) / 8) * a.tm));
#define ACT_GO(MB_) \
    if (act == MFMA_ACT_RELU2) hipLaunchKernelGGL((k_w16l_gemm<BF16, MB_, 2, MFMA_ACT_RELU2>), grid, dim3(256), 0, st, a); \
    else if (act == MFMA_ACT_GELU) hipLaunchKernelGGL((k_w16l_gemm<BF16, MB_, 2, MFMA_ACT_GELU>), grid, dim3(256), 0, st, a); \
    else if (act == MFMA_ACT_NONE) hipLaunchKernelGGL((k_w16l_gemm<BF16, MB_, 2, MFMA_ACT_NONE>), grid, dim3(256), 0, st, a); \
    else hipLaunchKernelGGL((k_w16l_gemm<BF16, MB_, 2, MFMA_ACT_XIELU>), grid, dim3(256), 0, st, a)
    if (mb == 2) { ACT_GO(2); }
    else if (mb == 4) { ACT_GO(4); }
    else { ACT_GO(8); }
#undef ACT_GO
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

// grouped: tiles [tm] of tile_rows (64 or 128) rows, `block` of them side by side on an XCD; x_rows: rows of x; act: MFMA_ACT_NONE, or MFMA_ACT_SWIGLU / _CLIPPED of the interleaved matrix, N / 2 wide
int w16l_grouped_launch(const void *w16m, size_t w_stride, const void *x, int ldx, size_t x_rows, const int *list, const void *tiles, int tm, int block, int tile_rows, int N, int K,
                        void *y, int ldy, int act, float act_alpha, float act_limit, hipStream_t st) {
    W16Args a = {};
    if (int rc = w16_fill(a, w16m, x, ldx, N, K, y, ldy)) return rc;
    PIE_REQUIRE(x_rows * ldx * 2 < (1ull << 32), PIE_E_SHAPE, "grouped GEMM: x too large");
    PIE_REQUIRE((tile_rows == 64 || tile_rows == 128) && (act == MFMA_ACT_NONE || N % 8 == 0), PIE_E_SHAPE, "grouped GEMM: bad tile or width");
    a.M = (int)x_rows, a.tm = tm, a.tiles = (const int4 *)tiles, a.list = list, a.w_stride = w_stride, a.act_alpha = act_alpha, a.act_limit = act_limit;
    a.bm = block;
    const dim3 grid((unsigned)(8 * ((tm + 8 * block - 1) / (8 * block)) * block * a.tn));
#define GRP_GO(MB_) \
    if (act == MFMA_ACT_SWIGLU) hipLaunchKernelGGL((k_w16l_gemm<BF16, MB_, 2, MFMA_ACT_SWIGLU, true>), grid, dim3(256), 0, st, a); \
    else if (act == MFMA_ACT_CLIPPED) hipLaunchKernelGGL((k_w16l_gemm<BF16, MB_, 2, MFMA_ACT_CLIPPED, true>), grid, dim3(256), 0, st, a); \
    else hipLaunchKernelGGL((k_w16l_gemm<BF16, MB_, 2, MFMA_ACT_NONE, true>), grid, dim3(256), 0, st, a)
    if (tile_rows == 64) { GRP_GO(2); } else { GRP_GO(4); }
#undef GRP_GO
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}
