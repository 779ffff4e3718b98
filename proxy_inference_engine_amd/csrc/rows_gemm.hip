// rows_gemm.hip -- the Linear of the layer-stack models: y[M, N] = x[M, K] . W[N, K]^T with the consumer's element-wise work in the epilogue.
//
// Few rows (a decode step, a short portion): the weights are read once and everything else is small.  A workgroup of eight waves owns
// 16 * NW output features; KW waves split K between them (NW * KW = 8).  A wave streams 1-KiB pieces of the W16M tiles (w16_gemm.hpp: 32
// features x 64 columns in MFMA operand order) -- half a tile row group per instruction, four 256-byte runs -- straight into the A operand of
// v_mfma_f32_16x16x32_bf16; the B operand is the matching 16 B of up to 16 rows of x, read through L2.  One row of x uses one of the 16 columns,
// which costs nothing: the matrix cores are idle either way.  The K-split partial sums meet in LDS.
//
// The same kernel runs batched over heads (per-head up- / down-projections), over a list of unlike matrices, grouped over the active experts of a mixture (row lists), and for
// any M (blockIdx.z walks 16 * NT rows at a time).
#include <algorithm>

#include "stack_types.hpp"

size_t w16m_size(int N, int K);

typedef __attribute__((ext_vector_type(8))) __bf16 mf_bf16x8;
typedef __attribute__((ext_vector_type(4))) float mf_f32x4;
typedef __attribute__((ext_vector_type(4))) u32 mf_u32x4;

namespace {

// What blockIdx.y selects: the matrix, its live rows, and how result rows map to x rows.
struct RowsWork {
    const char *w;
    const void *x;
    void *y;
    int N, K, ldx, ldy, count, row0;
    const int *rows;  // x row of local row i (nullptr: row0 + i)
    int xoff, yoff;
};
__device__ __forceinline__ bool rows_select(const RowsArgs &a, RowsWork &k) {
    k.w = a.m.w, k.x = a.m.x, k.y = a.m.y, k.N = a.m.N, k.K = a.m.K, k.ldx = a.m.ldx, k.ldy = a.m.ldy;
    k.count = a.M, k.row0 = 0, k.rows = a.rows, k.xoff = k.yoff = 0;
    const int b = blockIdx.y;
    if (a.n_mats) {
        const RowsMat &m = a.mats[b];
        k.w = m.w, k.x = m.x, k.y = m.y, k.N = m.N, k.K = m.K, k.ldx = m.ldx, k.ldy = m.ldy;
        return true;
    }
    if (a.shared.w && b == (int)gridDim.y - 1) {
        k.w = a.shared.w, k.x = a.shared.x, k.y = a.shared.y, k.N = a.shared.N, k.K = a.shared.K, k.ldx = a.shared.ldx, k.ldy = a.shared.ldy;
        return true;
    }
    if (a.active) {
        const int e = a.active[b];
        if (e < 0) return false;
        k.row0 = a.offset[e], k.count = a.offset[e + 1] - k.row0;
        if (a.gather) k.rows = a.list + k.row0;
        k.w += (size_t)e * a.w_batch;
        return true;
    }
    k.w += (size_t)b * a.w_batch, k.xoff = b * a.x_batch, k.yoff = b * a.y_batch;
    return true;
}

// One finished value (m: result row inside the group, n: feature); pair: the value of feature n + 1 (ROWS_SILU_MUL, ROWS_CLIP_MUL, ROWS_GELU_MUL)
template <class E>
__device__ __forceinline__ void rows_finish(const RowsArgs &a, const RowsWork &k, int m, int n, float v, float pair) {
    typedef typename E::type T;
    const size_t row = (size_t)(k.row0 + m);
    switch (a.epi) {
        case ROWS_STORE: ((T *)k.y)[row * k.ldy + k.yoff + n] = E::pack(v); break;
        case ROWS_SCALE_F32: ((float *)k.y)[row * k.ldy + k.yoff + n] = v * a.scale; break;
        case ROWS_RELU2: {
            const float r = fmaxf(v, 0.0f);
            ((T *)k.y)[row * k.ldy + n] = E::pack(r * r);
            break;
        }
        case ROWS_XIELU: ((T *)k.y)[row * k.ldy + n] = E::pack(xielu<sizeof(T) == 4>(v, a.act_alpha, a.act_limit)); break;
        case ROWS_SILU_MUL:
            if (!(n & 1)) ((T *)k.y)[row * k.ldy + (n >> 1)] = E::pack(v / (1.0f + expf(-v)) * pair);
            break;
        case ROWS_CLIP_MUL:
            if (!(n & 1)) ((T *)k.y)[row * k.ldy + (n >> 1)] = E::pack(clipped_glu(v, pair, a.act_alpha, a.act_limit));
            break;
        case ROWS_GELU_MUL:
            if (!(n & 1)) {
                if (a.bias) v += BF16::to_f32(a.bias[n]), pair += BF16::to_f32(a.bias[n + 1]);
                ((T *)k.y)[row * k.ldy + (n >> 1)] = E::pack(gelu_tanh<sizeof(T) == 4>(v) * pair);
            }
            break;
        case ROWS_GELU_SIDE: ((T *)k.y)[row * k.ldy + n] = E::pack(gelu_tanh<sizeof(T) == 4>(v) * BF16::to_f32(token_vector(a.side, row)[n])); break;
        case ROWS_SOFTCAP: ((float *)k.y)[row * k.ldy + n] = a.act_limit * stack_tanh<sizeof(T) == 4>(v * a.scale / a.act_limit); break;
        case ROWS_SPLIT:
            if (n < a.split) ((T *)k.y)[row * k.ldy + n] = E::pack(v);
            else a.y2[row * a.ldy2 + n - a.split] = v;
            break;
        case ROWS_RESIDUAL: {
            float *xp = a.res + row * a.ld_res + n;
            const float x = *xp + point_norm(a.post, n, v);
            *xp = x;
            ((T *)a.h)[row * a.ldh + n] = E::pack(point_norm(a.next, n, x));
            break;
        }
    }
}

__host__ __device__ __forceinline__ int rows_riders(const RowsArgs &a) { return (a.append.M > 0) + (a.cache.M > 0) + (a.rotate.M > 0); }
// the last blockIdx.y: what rides along
template <class E, int THREADS>
__device__ __forceinline__ bool rows_ride(const RowsArgs &a, float *red) {
    int i = (int)(gridDim.y - 1 - blockIdx.y);
    if (i >= rows_riders(a)) return false;
    if (blockIdx.z) return true;
    const bool append = a.append.M > 0 && i == 0;
    i -= a.append.M > 0;
    const bool cache = a.cache.M > 0 && i == 0;
    const int M = append ? a.append.M : cache ? a.cache.M : a.rotate.M;
    for (int m = blockIdx.x; m < M; m += gridDim.x) {
        if (append) latent_append_row<E, ElemF32, THREADS>(a.append, m, red);
        else if (cache) latent_cache_row<E, THREADS>(a.cache, m, red);
        else rotate_row<E, THREADS>(a.rotate, m);
        __syncthreads();
    }
    return true;
}

// NT: blocks of 16 rows of x; KW: waves along K; NN: blocks of 16 features per wave (two share the x operands); MERGE: x = the merged key splits of head
// blockIdx.y (RowsArgs::merge), put together in LDS by every workgroup of the head; NORM: RowsArgs::x_norm (every workgroup sees its rows whole)
template <int NT, int KW, int NN, bool MERGE = false, bool NORM = false>
__global__ void __launch_bounds__(512) k_rows_w16m(const RowsArgs a) {
    constexpr int NW = 8 / KW, U = NT >= 4 ? 2 : 4;
    constexpr int ST = 20;  // floats per (row, 16 features) line of the reduction image
    __shared__ __attribute__((aligned(16))) float s_red[8 * NN * NT * 16 * ST];
    __shared__ float s_ss[NORM ? 8 : 1][16];
    static_assert(!NORM || NT == 1, "norms: sixteen rows");
    if (rows_ride<ElemBF16, 512>(a, s_red)) return;
    __shared__ __attribute__((aligned(16))) u16 s_x[MERGE ? MERGE_ROWS * (MERGE_LDR + 64) : 8];
    const int ldx_lds = a.merge.ldr + 64;
    if constexpr (MERGE) {
        __shared__ float s_f[MERGE_ROWS][64];
        const int H = a.merge.H, M = a.merge.M, w = threadIdx.x >> 6;
        if (w < M) s_f[w][threadIdx.x & 63] = latent_split_weight(a.merge, (size_t)w * H + blockIdx.y, threadIdx.x & 63);
        __syncthreads();
        const int quads = ldx_lds / 4;
        for (int i = threadIdx.x; i < M * quads; i += 512) {
            const int m = i / quads, r = i % quads * 4;
            float4 v = make_float4(0, 0, 0, 0);  // (columns past the latent meet zero weights: zeros)
            if (r < a.merge.ldr) v = latent_merge4(a.merge, (size_t)m * H + blockIdx.y, r, [&](int s) { return s_f[m][s]; });
            *(uint2 *)(s_x + m * ldx_lds + r) = make_uint2(pack2<BF16>(v.x, v.y), pack2<BF16>(v.z, v.w));
        }
        __syncthreads();
    }
    RowsWork k;
    if (!rows_select(a, k)) return;
    const int i0 = blockIdx.z * 16 * NT;
    if (i0 >= k.count) return;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int wn = wave / KW, wk = wave % KW;
    const int t16 = (blockIdx.x * NW + wn) * NN;  // this wave's first block of 16 output features
    if ((int)blockIdx.x * NW * NN * 16 >= k.N) return;
    const int c = lane & 15, kq = lane >> 4;
    const int groups = (k.K + 63) >> 6, steps = 2 * groups;
    const bool live = t16 * 16 < k.N;  // (NN = 2: both blocks lie in one 32-row tile, which is stored whole)

    float ss = 0.0f;
    mf_f32x4 acc[NN][NT];
#pragma unroll
    for (int n = 0; n < NN; ++n)
#pragma unroll
        for (int t = 0; t < NT; ++t) acc[n][t] = (mf_f32x4){0.0f, 0.0f, 0.0f, 0.0f};
    if (live) {
        const char *wp = k.w + (size_t)(t16 >> 1) * groups * 4096 + ((kq >> 1) * 1024 + ((kq & 1) * 32 + (t16 & 1) * 16 + c) * 16);
        const u16 *xp[NT];
#pragma unroll
        for (int t = 0; t < NT; ++t) {
            int i = i0 + 16 * t + c;
            i = i < k.count ? i : k.count - 1;  // rows past the end repeat the last one (never stored)
            const int xr = k.rows ? k.rows[i] : k.row0 + i;
            xp[t] = MERGE ? s_x + xr * ldx_lds + 8 * kq : (const u16 *)k.x + (size_t)xr * k.ldx + k.xoff + 8 * kq;
        }
        auto fetch = [&](int s, mf_u32x4(&wv)[U][NN], mf_u32x4(&xv)[U][NT]) {
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int ss = s + u * KW, cl = ss < steps ? ss : steps - 1;
#pragma unroll
                for (int n = 0; n < NN; ++n) wv[u][n] = __builtin_nontemporal_load((const mf_u32x4 *)(wp + (size_t)cl * 2048 + n * 256));
#pragma unroll
                for (int t = 0; t < NT; ++t) xv[u][t] = *(const mf_u32x4 *)(xp[t] + 32 * cl);
            }
        };
        auto multiply = [&](int s, const mf_u32x4(&wv)[U][NN], const mf_u32x4(&xv)[U][NT]) {
#pragma unroll
            for (int u = 0; u < U; ++u)
#pragma unroll
                for (int n = 0; n < NN; ++n) {
                    mf_u32x4 w = wv[u][n];
                    if (s + u * KW >= steps) w = (mf_u32x4){0u, 0u, 0u, 0u};
                    if constexpr (NORM)
                        if (n == 0 && s + u * KW < steps && 32 * (s + u * KW) + 8 * kq < k.K)  // (what lies behind the row belongs to others; a row's padding to 8 is zero)
#pragma unroll
                            for (int i = 0; i < 4; ++i) ss = fmaf(lo_f32<BF16>(xv[u][0][i]), lo_f32<BF16>(xv[u][0][i]), fmaf(hi_f32<BF16>(xv[u][0][i]), hi_f32<BF16>(xv[u][0][i]), ss));
#pragma unroll
                    for (int t = 0; t < NT; ++t)
                        acc[n][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(mf_bf16x8, w), __builtin_bit_cast(mf_bf16x8, xv[u][t]), acc[n][t], 0, 0, 0);
                }
        };
        mf_u32x4 w0[U][NN], w1[U][NN], x0[U][NT], x1[U][NT];
        fetch(wk, w0, x0);
        for (int s = wk; s < steps; s += 2 * U * KW) {
            fetch(s + U * KW, w1, x1);
            multiply(s, w0, x0);
            fetch(s + 2 * U * KW, w0, x0);
            multiply(s + U * KW, w1, x1);
        }
    }
    if constexpr (NORM) {
        ss = xor32_sum(xor16_sum(ss));
        if (kq == 0) s_ss[wave][c] = ss;
    }
    // lane (kq, c) holds features 4 kq .. + 3 of row c
#pragma unroll
    for (int n = 0; n < NN; ++n)
#pragma unroll
        for (int t = 0; t < NT; ++t) *(mf_f32x4 *)(s_red + (((wave * NN + n) * NT + t) * 16 + c) * ST + 4 * kq) = acc[n][t];
    __syncthreads();
    const bool paired = a.epi == ROWS_SILU_MUL || a.epi == ROWS_CLIP_MUL || a.epi == ROWS_GELU_MUL;
    for (int id = threadIdx.x; id < NW * NN * NT * 256; id += 512) {
        const int nl = id & 15, ml = (id >> 4) % (16 * NT), wn2 = id / (256 * NT), w = wn2 / NN, nn = wn2 % NN;
        const int n = ((int)blockIdx.x * NW * NN + wn2) * 16 + nl, m = i0 + ml;
        if (n >= k.N || m >= k.count) continue;
        if (paired && (nl & 1)) continue;
        const float *r = s_red + (((w * KW * NN + nn) * NT + (ml >> 4)) * 16 + (ml & 15)) * ST + nl;
        float v = 0.0f, p = 0.0f;
#pragma unroll
        for (int q = 0; q < KW; ++q) v += r[q * NN * NT * 16 * ST];
        if (paired)
#pragma unroll
            for (int q = 0; q < KW; ++q) p += r[q * NN * NT * 16 * ST + 1];
        if constexpr (NORM) {
            float sum = 0.0f;
#pragma unroll
            for (int q = 0; q < KW; ++q) sum += s_ss[w * KW + q][ml];
            v *= 1.0f / sqrtf(sum / (float)k.K + a.x_eps);
        }
        rows_finish<ElemBF16>(a, k, m, n, v, p);
    }
}

// fp32: one output per thread, 16 features x 16 rows per workgroup, both operands through LDS
__global__ void __launch_bounds__(256) k_rows_f32(const RowsArgs a) {
    __shared__ float s_w[16][65], s_x[16][65], s_v[16][17];
    if (rows_ride<ElemF32, 256>(a, s_v[0])) return;
    RowsWork k;
    if (!rows_select(a, k)) return;
    const int i0 = blockIdx.z * 16, n0 = blockIdx.x * 16;
    if (i0 >= k.count || n0 >= k.N) return;
    const int tn = threadIdx.x & 15, tm = threadIdx.x >> 4;
    const int Kp = (k.K + 63) & ~63;
    float acc = 0.0f;
    for (int k0 = 0; k0 < Kp; k0 += 64) {
        for (int id = threadIdx.x; id < 1024; id += 256) {
            const int r = id >> 6, c = id & 63;
            s_w[r][c] = n0 + r < k.N ? ((const float *)k.w)[(size_t)(n0 + r) * Kp + k0 + c] : 0.0f;
            int i = i0 + r;
            i = i < k.count ? i : k.count - 1;
            const int xr = k.rows ? k.rows[i] : k.row0 + i;
            s_x[r][c] = k0 + c < k.K ? ((const float *)k.x)[(size_t)xr * k.ldx + k.xoff + k0 + c] : 0.0f;
        }
        __syncthreads();
#pragma unroll 16
        for (int c = 0; c < 64; ++c) acc = fmaf(s_w[tn][c], s_x[tm][c], acc);
        __syncthreads();
    }
    s_v[tm][tn] = acc;
    __syncthreads();
    const int n = n0 + tn, m = i0 + tm;
    if (n < k.N && m < k.count) rows_finish<ElemF32>(a, k, m, n, acc, s_v[tm][tn < 15 ? tn + 1 : 15]);
}

template <int NT, int NN>
int rows_go(const RowsArgs &a, int n_max, int k_max, int batches, hipStream_t st) {
    const int steps = 2 * ((k_max + 63) / 64), tiles = (n_max + 16 * NN - 1) / (16 * NN);
    const int z = (a.M + 16 * NT - 1) / (16 * NT);  // (grouped: most experts have few rows, their later z leave at once)
    // waves along K: enough steps for each, and enough workgroups for the chip
    int kw = steps >= 32 ? 8 : steps >= 16 ? 4 : steps >= 8 ? 2 : 1;
    while (kw < 8 && steps >= 2 * kw && (size_t)((tiles + 8 / kw - 1) / (8 / kw)) * batches * z < 256) kw *= 2;
    const dim3 grid((unsigned)((tiles + 8 / kw - 1) / (8 / kw)), (unsigned)(batches + rows_riders(a)), (unsigned)z);
    if (a.x_norm) {
        if (kw == 8) hipLaunchKernelGGL((k_rows_w16m<1, 8, 1, false, true>), grid, dim3(512), 0, st, a);
        else if (kw == 4) hipLaunchKernelGGL((k_rows_w16m<1, 4, 1, false, true>), grid, dim3(512), 0, st, a);
        else if (kw == 2) hipLaunchKernelGGL((k_rows_w16m<1, 2, 1, false, true>), grid, dim3(512), 0, st, a);
        else hipLaunchKernelGGL((k_rows_w16m<1, 1, 1, false, true>), grid, dim3(512), 0, st, a);
    } else if (a.merge.splits > 0) {
        if (kw == 8) hipLaunchKernelGGL((k_rows_w16m<1, 8, 1, true>), grid, dim3(512), 0, st, a);
        else if (kw == 4) hipLaunchKernelGGL((k_rows_w16m<1, 4, 1, true>), grid, dim3(512), 0, st, a);
        else if (kw == 2) hipLaunchKernelGGL((k_rows_w16m<1, 2, 1, true>), grid, dim3(512), 0, st, a);
        else hipLaunchKernelGGL((k_rows_w16m<1, 1, 1, true>), grid, dim3(512), 0, st, a);
    } else if (kw == 8) hipLaunchKernelGGL((k_rows_w16m<NT, 8, NN>), grid, dim3(512), 0, st, a);
    else if (kw == 4) hipLaunchKernelGGL((k_rows_w16m<NT, 4, NN>), grid, dim3(512), 0, st, a);
    else if (kw == 2) hipLaunchKernelGGL((k_rows_w16m<NT, 2, NN>), grid, dim3(512), 0, st, a);
    else hipLaunchKernelGGL((k_rows_w16m<NT, 1, NN>), grid, dim3(512), 0, st, a);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

__global__ void __launch_bounds__(256) k_pack_f32(const u16 *w, int N, int K, int Kp, float *out) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= (size_t)N * Kp) return;
    const int n = (int)(i / Kp), c = (int)(i % Kp);
    out[i] = c < K ? BF16::to_f32(w[(size_t)n * K + c]) : 0.0f;
}

}  // namespace

size_t rows_weight_bytes(int dtype, int N, int K) {
    return dtype == PIE_F32 ? (size_t)N * ((K + 63) & ~63) * 4 : w16m_size(N, K);
}

int rows_gemm_launch(int dtype, const RowsArgs &a, int batches, hipStream_t st) {
    if (a.M <= 0 || batches <= 0) return PIE_OK;
    PIE_REQUIRE(a.n_mats || (a.m.N > 0 && a.m.K > 0), PIE_E_SHAPE, "row-wise Linear: empty matrix");
    PIE_REQUIRE(batches < 65535 && (!rows_riders(a) || !(a.shared.w || a.active)), PIE_E_SHAPE, "row-wise Linear: too many batches");
    PIE_REQUIRE(a.n_mats == 0 || (a.n_mats == batches && a.n_mats <= ROWS_LIST && !rows_riders(a) && !a.shared.w && !a.active && !a.rows && a.merge.splits <= 0 && !a.x_norm), PIE_E_ARG,
                "row-wise Linear: a list of matrices is a launch of its own");
    int n_max = a.shared.w && a.shared.N > a.m.N ? a.shared.N : a.m.N, k_max = a.shared.w && a.shared.K > a.m.K ? a.shared.K : a.m.K;
    for (int i = 0; i < a.n_mats; ++i) {
        const RowsMat &m = a.mats[i];
        PIE_REQUIRE(m.N > 0 && m.K > 0 && m.ldx % 8 == 0 && pie_aligned(m.x, 16) && pie_aligned(m.w, 16), PIE_E_ALIGN, "row-wise Linear: 16-byte alignment required");
        n_max = i ? std::max(n_max, m.N) : m.N, k_max = i ? std::max(k_max, m.K) : m.K;
    }
    PIE_REQUIRE(!a.x_norm || (dtype == PIE_BF16 && a.M <= 16 && batches == 1 && !a.active && !a.shared.w && !a.rows && a.merge.splits <= 0), PIE_E_SHAPE, "row-wise Linear: too many rows to norm on the way in");
    if (dtype == PIE_F32) {
        const dim3 grid((unsigned)((n_max + 15) / 16), (unsigned)(batches + rows_riders(a)), (unsigned)((a.M + 15) / 16));
        hipLaunchKernelGGL(k_rows_f32, grid, dim3(256), 0, st, a);
        PIE_LAUNCH_CHECK();
        return PIE_OK;
    }
    PIE_REQUIRE(a.merge.splits <= 64 && (a.merge.splits <= 0 || (a.merge.M == a.M && a.M <= MERGE_ROWS && a.merge.ldr <= MERGE_LDR && a.merge.ldr % 8 == 0 && !a.active && !a.rows)), PIE_E_SHAPE,
                "row-wise Linear: too many rows or columns to merge key splits on the way in");
    PIE_REQUIRE(a.m.ldx % 8 == 0 && a.x_batch % 8 == 0 && pie_aligned(a.m.x, 16) && pie_aligned(a.m.w, 16), PIE_E_ALIGN, "row-wise Linear: 16-byte alignment required");
    int n_all = batches == 1 ? n_max : 0;
    for (int i = 0; i < a.n_mats; ++i) n_all += a.mats[i].N;
    const bool narrow = (long)batches * n_max <= 16 * 64 && !a.merge.splits;  // so few workgroups that they should not all read all rows
    if (a.M <= 16 || a.active || narrow) return rows_go<1, 1>(a, n_max, k_max, batches, st);
    const bool wide = n_all >= 32 * 140;  // two feature blocks per wave where half as many workgroups still fill most of the chip
    if (a.M <= 32) return wide ? rows_go<2, 2>(a, n_max, k_max, batches, st) : rows_go<2, 1>(a, n_max, k_max, batches, st);
    return wide ? rows_go<4, 2>(a, n_max, k_max, batches, st) : rows_go<4, 1>(a, n_max, k_max, batches, st);
}

extern "C" {

size_t pie_stack_weight_bytes(int dtype, int N, int K) {
    return N > 0 && K > 0 && (dtype == PIE_BF16 || dtype == PIE_F32) ? rows_weight_bytes(dtype, N, K) : 0;
}

int pie_stack_pack_weight(const void *w, int N, int K, int dtype, void *packed, void *stream) {
    PIE_REQUIRE(w && packed, PIE_E_ARG, "pie_stack_pack_weight: null pointer");
    PIE_REQUIRE(N > 0 && K > 0, PIE_E_SHAPE, "pie_stack_pack_weight: empty matrix");
    if (dtype == PIE_BF16) return pie_repack_w16m(w, N, K, PIE_BF16, packed, stream);
    PIE_REQUIRE(dtype == PIE_F32, PIE_E_ARG, "pie_stack_pack_weight: dtype must be PIE_BF16 or PIE_F32");
    const int Kp = (K + 63) & ~63;
    hipLaunchKernelGGL(k_pack_f32, dim3((unsigned)(((size_t)N * Kp + 255) / 256)), dim3(256), 0, (hipStream_t)stream, (const u16 *)w, N, K, Kp, (float *)packed);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

}  // extern "C"
