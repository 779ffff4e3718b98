// row_update.hip -- what stands between two sublayers when a norm needs the whole row: x += post(y), or x = post(alpha x + y); h = next(x).
//
// One workgroup per row.  y is a sublayer's output (plus a bias), or the weighted sum of a row's experts; the row stays in registers from the first read to
// the last store, so the norms' sums cost one exchange through LDS each and x, y and h pass through memory once.
//
// In front of a mixer that reads every token mixed with its predecessor, the mixes are made of the new x: by the same workgroup where every run is one row (the predecessor is
// the sequence's state), by a launch behind it (k_token_mix) where runs are longer.
//
// Few rows in front of a mixture: the workgroup goes on with its row's router logits (the row is in LDS, a wave per expert), chooses the experts, and the
// last workgroup to arrive makes the row lists -- the router, the choice and the lists are no launches of their own.
#include "route.hpp"
#include "row_norm.hpp"

namespace {

// the router's logits of the row in s_row; EB: experts of a wave in flight (the weights come from memory, and a wave has few of them)
template <int EB, int NW>
__device__ __forceinline__ void row_logits(const RowUpdateArgs &a, const float *s_row, float *s_z, int W8) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    for (int e0 = wave; e0 < a.experts; e0 += EB * NW) {
        float z[EB];
#pragma unroll
        for (int i = 0; i < EB; ++i) z[i] = 0.0f;
#pragma unroll 4
        for (int k = lane * 8; k < W8; k += 512) {
            uint4 v[EB];
#pragma unroll
            for (int i = 0; i < EB; ++i) v[i] = *(const uint4 *)(a.router + (size_t)min(e0 + i * NW, a.experts - 1) * W8 + k);
            const float4 h0 = *(const float4 *)(s_row + k), h1 = *(const float4 *)(s_row + k + 4);
#pragma unroll
            for (int i = 0; i < EB; ++i) {
                z[i] = fmaf(lo_f32<BF16>(v[i].x), h0.x, fmaf(hi_f32<BF16>(v[i].x), h0.y, fmaf(lo_f32<BF16>(v[i].y), h0.z, fmaf(hi_f32<BF16>(v[i].y), h0.w, z[i]))));
                z[i] = fmaf(lo_f32<BF16>(v[i].z), h1.x, fmaf(hi_f32<BF16>(v[i].z), h1.y, fmaf(lo_f32<BF16>(v[i].w), h1.z, fmaf(hi_f32<BF16>(v[i].w), h1.w, z[i]))));
            }
        }
#pragma unroll
        for (int i = 0; i < EB; ++i) {
            const float sum = lanes_sum(z[i]);
            if (lane == 0 && e0 + i * NW < a.experts) s_z[e0 + i * NW] = sum;
        }
    }
}

// xv: next(x) of row blockIdx.x, quads as in k_row_update
template <int THREADS, int NQ>
__device__ __forceinline__ void row_route(const RowUpdateArgs &a, const float (&xv)[NQ][4]) {
    extern __shared__ __attribute__((aligned(16))) float s_dyn[];  // [W rounded up to 8] the row, [experts] logits, [2 * experts] list counters
    const int W8 = (a.W + 7) & ~7, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, m = blockIdx.x;
    float *s_z = s_dyn + W8;
    int *s_cnt = (int *)(s_z + a.experts);
    __shared__ int s_last;
    const RouteLayer L = *a.route;
    float corr[ROUTE_KEPT];
    route_corrections(L, lane, corr);
#pragma unroll
    for (int q = 0; q < NQ; ++q) {
        const int n = threadIdx.x * 4 + 4 * THREADS * q;
        if (n < W8) *(float4 *)(s_dyn + n) = make_float4(xv[q][0], xv[q][1], xv[q][2], xv[q][3]);  // (zeros past W)
    }
    __syncthreads();
    constexpr int NW = THREADS / 64;
    if (a.experts <= NW) row_logits<1, NW>(a, s_dyn, s_z, W8);
    else if (a.experts <= 2 * NW) row_logits<2, NW>(a, s_dyn, s_z, W8);
    else row_logits<4, NW>(a, s_dyn, s_z, W8);
    __syncthreads();
    if (wave == 0) {
        route_pick(L, s_z, lane, corr, [&](int k, int e, float w) {
            if (lane) return;
            const size_t i = (size_t)m * L.top + k;
            __hip_atomic_store(L.chosen + i, e, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);  // (seen by whichever workgroup arrives last, on any XCD)
            L.weight[i] = w;
        });
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        if (lane == 0) s_last = __hip_atomic_fetch_add(a.arrived, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == (int)gridDim.x - 1;
    }
    __syncthreads();
    if (!s_last) return;
    if (threadIdx.x == 0) __hip_atomic_store(a.arrived, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    route_lists(L, a.M, s_cnt, [&](int i) { return __hip_atomic_load(L.chosen + i, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT); }, 0, 0, 0);
}

// the mixes of one quad of row m's columns; before: the predecessor's
template <class E>
__device__ __forceinline__ void token_mix4(const TokenMixArgs &a, size_t m, size_t M, int n, int W, const float (&x)[4], const float (&before)[4]) {
    typedef typename E::type T;
#pragma unroll
    for (int s = 0; s < TIME_MIXES; ++s) {
        const float4 mu = *(const float4 *)(a.mu + (size_t)s * a.ldmu + n);  // (padded)
        const float y[4] = {fmaf(before[0] - x[0], mu.x, x[0]), fmaf(before[1] - x[1], mu.y, x[1]), fmaf(before[2] - x[2], mu.z, x[2]), fmaf(before[3] - x[3], mu.w, x[3])};
        T *out = (T *)a.out + (s * M + m) * a.ldo + n;
        if (n + 4 <= W) {
            if constexpr (sizeof(T) == 2) *(uint2 *)out = make_uint2(pack2<BF16>(y[0], y[1]), pack2<BF16>(y[2], y[3]));
            else *(float4 *)out = make_float4(y[0], y[1], y[2], y[3]);
        } else
            for (int i = 0; i < W - n; ++i) out[i] = E::pack(y[i]);
    }
}
__device__ __forceinline__ float *token_mix_state(const TokenMixArgs &a, int m) {
    return a.state + min((unsigned)a.slots[min(a.row_seq[m], a.n_seqs - 1)], (unsigned)a.n_slots - 1u) * a.slot_floats;
}

// A thread takes four columns of a row.  The workgroup of a run's first row reads what the state holds and then writes the run's last row there.
template <class E>
__global__ void __launch_bounds__(256) k_token_mix(const TokenMixArgs a, const float *x, int ldx, int W) {
    const int n = (blockIdx.x * 256 + threadIdx.x) * 4, m = blockIdx.y;
    if (n >= W) return;
    const bool first = m == 0 || a.row_seq[m - 1] != a.row_seq[m];
    const float4 v = *(const float4 *)(x + (size_t)m * ldx + n);
    float4 p = make_float4(0, 0, 0, 0);
    if (!first) p = *(const float4 *)(x + (size_t)(m - 1) * ldx + n);
    else {
        float *held = token_mix_state(a, m) + n;
        if (a.pos[m] > 0) p = *(const float4 *)held;
        int last = m;
        for (int r = 0; r < a.n_runs; ++r)
            if (a.runs[r].row0 == m) last = m + a.runs[r].n_rows - 1;
        *(float4 *)held = *(const float4 *)(x + (size_t)last * ldx + n);
    }
    const float xv[4] = {v.x, v.y, v.z, v.w}, pv[4] = {p.x, p.y, p.z, p.w};
    token_mix4<E>(a, m, gridDim.y, n, W, xv, pv);
}

template <class E, int THREADS, int NQ, bool ROUTE = false>
__global__ void __launch_bounds__(THREADS) k_row_update(const RowUpdateArgs a) {
    typedef typename E::type T;
    __shared__ float red[2][THREADS / 64];
    const size_t m = blockIdx.x;
    const int n0 = threadIdx.x * 4;
    float *x = a.x + m * a.ldx;
    float xv[NQ][4], y[NQ][4];
#pragma unroll
    for (int q = 0; q < NQ; ++q) {
        const int n = n0 + 4 * THREADS * q;
        float4 v = make_float4(0, 0, 0, 0);
        if (n < a.W) v = *(const float4 *)(x + n);
        xv[q][0] = v.x, xv[q][1] = v.y, xv[q][2] = v.z, xv[q][3] = v.w;
#pragma unroll
        for (int i = 0; i < 4; ++i) y[q][i] = 0.0f;
    }
    if (a.y) {
        if (a.place) {
            constexpr int U = NQ >= 4 ? 4 : 8;  // slots in flight
            const float share = 1.0f / (float)a.top;
            for (int s0 = 0; s0 < a.top; s0 += U) {
                float w[U];
                int at[U];
#pragma unroll
                for (int u = 0; u < U; ++u) {
                    const size_t i = m * a.top + min(s0 + u, a.top - 1);
                    at[u] = a.place[i], w[u] = s0 + u < a.top ? (a.weight ? a.weight[i] : share) : 0.0f;
                }
#pragma unroll
                for (int q = 0; q < NQ; ++q) {
                    const int n = n0 + 4 * THREADS * q;
                    if (n >= a.W) break;
                    float4 v[U];
#pragma unroll
                    for (int u = 0; u < U; ++u) v[u] = load_quad(a.y, a.y32, at[u], n, a.W, a.ldy);
#pragma unroll
                    for (int u = 0; u < U; ++u)
                        y[q][0] = fmaf(w[u], v[u].x, y[q][0]), y[q][1] = fmaf(w[u], v[u].y, y[q][1]), y[q][2] = fmaf(w[u], v[u].z, y[q][2]), y[q][3] = fmaf(w[u], v[u].w, y[q][3]);
                }
            }
        } else {
#pragma unroll
            for (int q = 0; q < NQ; ++q) {
                const int n = n0 + 4 * THREADS * q;
                if (n >= a.W) break;
                const float4 v = load_quad(a.y, a.y32, m, n, a.W, a.ldy);
                y[q][0] = v.x, y[q][1] = v.y, y[q][2] = v.z, y[q][3] = v.w;
                if (a.bias)
#pragma unroll
                    for (int i = 0; i < 4; ++i) y[q][i] += BF16::to_f32(a.bias[min(n + i, a.W - 1)]);
            }
        }
#pragma unroll
        for (int q = 0; q < NQ; ++q)  // columns past the row's end: nothing
#pragma unroll
            for (int i = 0; i < 4; ++i)
                if (n0 + 4 * THREADS * q + i >= a.W) y[q][i] = xv[q][i] = 0.0f;
        if (a.after) {
#pragma unroll
            for (int q = 0; q < NQ; ++q)
#pragma unroll
                for (int i = 0; i < 4; ++i) y[q][i] = fmaf(a.alpha, xv[q][i], y[q][i]), xv[q][i] = 0.0f;
        }
        norm_row<THREADS, NQ>(a.post, a.W, y, red[0]);
#pragma unroll
        for (int q = 0; q < NQ; ++q) {
            const int n = n0 + 4 * THREADS * q;
#pragma unroll
            for (int i = 0; i < 4; ++i) xv[q][i] += y[q][i];
            if (n + 4 <= a.W) *(float4 *)(x + n) = make_float4(xv[q][0], xv[q][1], xv[q][2], xv[q][3]);
            else
                for (int i = 0; i < a.W - n; ++i) x[n + i] = xv[q][i];
        }
    } else {
#pragma unroll
        for (int q = 0; q < NQ; ++q)
#pragma unroll
            for (int i = 0; i < 4; ++i)
                if (n0 + 4 * THREADS * q + i >= a.W) xv[q][i] = 0.0f;
    }
    if (a.mix.mu) {
        float *held = token_mix_state(a.mix, (int)m);
        const bool fresh = a.mix.pos[m] == 0;
#pragma unroll
        for (int q = 0; q < NQ; ++q) {
            const int n = n0 + 4 * THREADS * q;
            if (n >= a.W) break;
            const float4 p = fresh ? make_float4(0, 0, 0, 0) : *(const float4 *)(held + n);
            const float pv[4] = {p.x, p.y, p.z, p.w};
            token_mix4<E>(a.mix, m, gridDim.x, n, a.W, xv[q], pv);
            *(float4 *)(held + n) = make_float4(xv[q][0], xv[q][1], xv[q][2], xv[q][3]);
        }
    }
    norm_row<THREADS, NQ>(a.next, a.W, xv, red[1]);
    T *h = (T *)a.h + m * a.ldh;
#pragma unroll
    for (int q = 0; q < NQ; ++q) {
        const int n = n0 + 4 * THREADS * q;
        if (n + 4 <= a.W) {
            if constexpr (sizeof(T) == 2) *(uint2 *)(h + n) = make_uint2(pack2<BF16>(xv[q][0], xv[q][1]), pack2<BF16>(xv[q][2], xv[q][3]));
            else *(float4 *)(h + n) = make_float4(xv[q][0], xv[q][1], xv[q][2], xv[q][3]);
        } else
            for (int i = 0; i < a.W - n; ++i) h[n + i] = E::pack(xv[q][i]);
    }
    if constexpr (ROUTE) row_route<THREADS, NQ>(a, xv);
}

template <class E>
void row_go(const RowUpdateArgs &a, hipStream_t st) {
    const dim3 grid((unsigned)a.M);
    if (a.route) {  // (always sixteen waves: they share the experts)
        const size_t lds = ((size_t)((a.W + 7) & ~7) + 3 * a.experts) * 4;
#define ROW_GO(T_, Q_) hipLaunchKernelGGL((k_row_update<E, T_, Q_, true>), grid, dim3(T_), lds, st, a)
        if (a.W <= 4096) ROW_GO(1024, 1);
        else ROW_GO(1024, 4);
#undef ROW_GO
        return;
    }
#define ROW_GO(T_, Q_) hipLaunchKernelGGL((k_row_update<E, T_, Q_>), grid, dim3(T_), 0, st, a)
    if (a.W <= 256) ROW_GO(64, 1);
    else if (a.W <= 1024) ROW_GO(256, 1);
    else if (a.M >= 512 && a.W <= 4096) {  // many rows: fewer, longer-lived workgroups per row
        if (a.W <= 2048) ROW_GO(256, 2);
        else ROW_GO(256, 4);
    } else if (a.W <= 2048) ROW_GO(512, 1);
    else if (a.W <= 4096) ROW_GO(1024, 1);
    else if (a.W <= 8192) ROW_GO(1024, 2);
    else if (a.W <= 16384) ROW_GO(1024, 4);
    else ROW_GO(1024, 8);
#undef ROW_GO
}

}  // namespace

int row_update_launch(int dtype, const RowUpdateArgs &a, hipStream_t st) {
    if (a.M <= 0) return PIE_OK;
    PIE_REQUIRE(a.W > 0 && a.W <= ROW_UPDATE_MAX_WIDTH, PIE_E_SHAPE, "row update: widths up to 32768");
    PIE_REQUIRE(a.ldx % 4 == 0 && a.ldh % 4 == 0 && (!a.y32 || a.ldy % 4 == 0), PIE_E_ALIGN, "row update: row strides must be multiples of 4");
    PIE_REQUIRE(!a.route || (a.router && a.arrived && a.experts > 0 && ((size_t)a.W + 8 + 3 * a.experts) * 4 <= 64 * 1024 - 1024 && a.W <= 16384), PIE_E_SHAPE, "row update: too wide to route beside");
    if (dtype == PIE_F32) row_go<ElemF32>(a, st);
    else row_go<ElemBF16>(a, st);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

int token_mix_launch(int dtype, const TokenMixArgs &a, const float *x, int ldx, int M, int W, hipStream_t st) {
    if (M <= 0) return PIE_OK;
    PIE_REQUIRE(a.mu && a.state && a.out && a.slots && a.runs && a.n_runs > 0, PIE_E_ARG, "token mixes: missing operand");
    PIE_REQUIRE(W > 0 && M <= 65535 && ldx % 4 == 0 && a.ldo % 4 == 0 && a.ldmu % 4 == 0 && a.ldmu >= ((W + 3) & ~3) && a.slot_floats % 4 == 0, PIE_E_ALIGN, "token mixes: row strides must be multiples of 4");
    const dim3 grid((unsigned)((W + 1023) / 1024), (unsigned)M);
    if (dtype == PIE_F32) hipLaunchKernelGGL(k_token_mix<ElemF32>, grid, dim3(256), 0, st, a, x, ldx, W);
    else hipLaunchKernelGGL(k_token_mix<ElemBF16>, grid, dim3(256), 0, st, a, x, ldx, W);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}
