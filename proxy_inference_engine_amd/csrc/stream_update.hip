// stream_update.hip -- what stands between two sublayers of a model with several residual streams (hyper-connections): x_t <- sum_s mix[s][t] x_s + out[t] y,
// h = next(sum_s in[s] x_s) -- and, in front of a mixer, a causal convolution over time on every channel of h.
//
// One workgroup per row.  A thread takes a quad of columns of all streams at a time, so every stream is read and written once and only the weighted sum (what
// the norm needs) stays in registers.  The streams' first values come from the embedding in the same launch (token + bigram + position vectors).
// The convolution reads the rows in front: where every run is a single row these are the sequence's state alone and the same workgroup takes it, a pass with
// longer runs has a launch of its own for it (conv_launch) behind the plain h.  h is rounded to the stack's dtype before it is convolved, in both.
#include "row_norm.hpp"

namespace {

template <class E>
__device__ __forceinline__ float4 load_h4(const typename E::type *p) {
    if constexpr (sizeof(typename E::type) == 4) return *(const float4 *)p;
    else {
        const uint2 v = *(const uint2 *)p;
        return make_float4(lo_f32<BF16>(v.x), hi_f32<BF16>(v.x), lo_f32<BF16>(v.y), hi_f32<BF16>(v.y));
    }
}
template <class E>
__device__ __forceinline__ void store_h4(typename E::type *p, const float4 &v) {
    if constexpr (sizeof(typename E::type) == 4) *(float4 *)p = v;
    else *(uint2 *)p = make_uint2(pack2<BF16>(v.x, v.y), pack2<BF16>(v.z, v.w));
}
template <class E>
__device__ __forceinline__ float round_h(float v) { return sizeof(typename E::type) == 4 ? v : round_T<BF16>(v); }
__device__ __forceinline__ float4 fma4(const float4 &a, const float4 &b, const float4 &c) { return make_float4(fmaf(a.x, b.x, c.x), fmaf(a.y, b.y, c.y), fmaf(a.z, b.z, c.z), fmaf(a.w, b.w, c.w)); }
__device__ __forceinline__ float4 fma1(float a, const float4 &b, const float4 &c) { return make_float4(fmaf(a, b.x, c.x), fmaf(a, b.y, c.y), fmaf(a, b.z, c.z), fmaf(a, b.w, c.w)); }

__device__ __forceinline__ float *conv_state(const ConvArgs &a, int m) {
    return a.state + min((unsigned)a.slots[min(a.row_seq[m], a.n_seqs - 1)], (unsigned)a.n_slots - 1u) * a.slot_floats;
}

// four columns of a bf16 table row, zeros past W
__device__ __forceinline__ float4 table4(const u16 *row, int n, int W) {
    if (!(W & 3)) {
        const uint2 t = *(const uint2 *)(row + n);
        return make_float4(lo_f32<BF16>(t.x), hi_f32<BF16>(t.x), lo_f32<BF16>(t.y), hi_f32<BF16>(t.y));
    }
    float e[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) e[i] = n + i < W ? BF16::to_f32(row[n + i]) : 0.0f;
    return make_float4(e[0], e[1], e[2], e[3]);
}

// the rows of the three tables that row m's embedding is the sum of; carries the sequence's previous token
struct EmbedRows {
    const u16 *token, *bigram, *position;
};
__device__ __forceinline__ EmbedRows embed_rows(const StreamUpdateArgs &a, int m) {
    const StackEmbed &e = a.embed;
    const ConvArgs &c = a.conv;
    const int id = min(max(e.ids[m], 0), e.vocab - 1), t = c.pos[m];
    EmbedRows r = {e.table + (size_t)id * a.W, nullptr, e.positions ? e.positions + (size_t)min(max(t, 0), e.max_positions - 1) * a.W : nullptr};
    if (!e.bigram) return r;
    const bool first = m == 0 || c.row_seq[m - 1] != c.row_seq[m];  // of its run
    int *held = nullptr, prev = 0;
    if (first) {
        held = (int *)(e.prev + min((unsigned)c.slots[min(c.row_seq[m], c.n_seqs - 1)], (unsigned)c.n_slots - 1u) * c.slot_floats);
        prev = *held;
    } else prev = e.ids[m - 1];
    long long row = e.buckets;
    if (t > 0) {
        row = ((long long)min(max(prev, 0), e.vocab - 1) * e.mul_prev + (long long)id * e.mul_cur) % e.buckets;
        if (row < 0) row += e.buckets;
    }
    r.bigram = e.bigram + (size_t)row * a.W;
    if (first) {  // the run's last token is the next pass's previous one
        __syncthreads();  // (everyone has read the old one)
        int last = m;
        if (!a.single) {
            __shared__ int s_last;
            for (int i = threadIdx.x; i < c.n_runs; i += blockDim.x)
                if (c.runs[i].row0 == m) s_last = m + c.runs[i].n_rows - 1;
            __syncthreads();
            last = s_last;
        }
        if (threadIdx.x == 0) *held = min(max(e.ids[last], 0), e.vocab - 1);
    }
    return r;
}

// NS: streams at most (a.S of them)
template <class E, int THREADS, int NQ, int NS>
__global__ void __launch_bounds__(THREADS) k_stream_update(const StreamUpdateArgs a) {
    typedef typename E::type T;
    __shared__ float red[THREADS / 64];
    const int m = blockIdx.x, S = NS <= 4 ? NS : a.S, W = a.W;
    const int n0 = threadIdx.x * 4;
    float *x = a.x + (size_t)m * S * a.ldx;
    EmbedRows rows = {nullptr, nullptr, nullptr};
    if (a.embed.ids) rows = embed_rows(a, m);
    float u[NQ][4];
#pragma unroll
    for (int q = 0; q < NQ; ++q) {
        const int n = n0 + 4 * THREADS * q;
        float4 sum = make_float4(0, 0, 0, 0);
        if (n < W) {
            float4 v[NS];
            if (a.embed.ids) {
                float4 b = table4(rows.token, n, W);
                b = make_float4(b.x * a.embed.scale, b.y * a.embed.scale, b.z * a.embed.scale, b.w * a.embed.scale);
                if (rows.bigram) b = fma1(1.0f, table4(rows.bigram, n, W), b);
                if (rows.position) b = fma1(1.0f, table4(rows.position, n, W), b);
#pragma unroll
                for (int s = 0; s < NS; ++s)
                    if (s < S) v[s] = b, *(float4 *)(x + s * a.ldx + n) = b;
            } else {
#pragma unroll
                for (int s = 0; s < NS; ++s) v[s] = s < S ? *(const float4 *)(x + s * a.ldx + n) : make_float4(0, 0, 0, 0);
                if (a.y) {
                    float4 y = load_quad(a.y, a.y32, m, n, W, a.ldy), w[NS];
#pragma unroll
                    for (int t = 0; t < NS; ++t) {
                        if (t >= S) continue;
                        w[t] = make_float4(0, 0, 0, 0);
                        w[t] = fma1(a.out[t], y, w[t]);
#pragma unroll
                        for (int s = 0; s < NS; ++s)
                            if (s < S) w[t] = fma1(a.mix[s * S + t], v[s], w[t]);
                        *(float4 *)(x + t * a.ldx + n) = w[t];
                    }
#pragma unroll
                    for (int s = 0; s < NS; ++s) v[s] = s < S ? w[s] : make_float4(0, 0, 0, 0);
                }
            }
#pragma unroll
            for (int s = 0; s < NS; ++s)
                if (s < S) sum = fma1(a.in ? a.in[s] : 1.0f, v[s], sum);
        }
        u[q][0] = sum.x, u[q][1] = sum.y, u[q][2] = sum.z, u[q][3] = sum.w;
#pragma unroll
        for (int i = 0; i < 4; ++i)
            if (n + i >= W) u[q][i] = 0.0f;
    }
    norm_row<THREADS, NQ>(a.next, W, u, red);
    T *h = (T *)a.h + (size_t)m * a.ldh;
    const ConvArgs &c = a.conv;
    const bool conv = a.single && c.w;
    const int taps = c.taps, W4 = (W + 3) & ~3;
    float *held = nullptr;
    bool fresh = false;
    if (conv && taps > 1) held = conv_state(c, m), fresh = c.pos[m] == 0;
#pragma unroll
    for (int q = 0; q < NQ; ++q) {
        const int n = n0 + 4 * THREADS * q;
        if (n >= W) break;
        float4 y = make_float4(u[q][0], u[q][1], u[q][2], u[q][3]);
        if (conv) {
            const float4 r = make_float4(round_h<E>(y.x), round_h<E>(y.y), round_h<E>(y.z), round_h<E>(y.w));
            y = fma4(*(const float4 *)(c.w + (size_t)(taps - 1) * c.ldw + n), r, r);
            constexpr int NT = 3;  // inputs in flight
            for (int j0 = 0; j0 < taps - 1; j0 += NT) {
                float4 v[NT], w[NT];
#pragma unroll
                for (int j = 0; j < NT; ++j) {
                    const int i = min(j0 + j, taps - 2);
                    v[j] = *(const float4 *)(held + (size_t)i * W4 + n), w[j] = *(const float4 *)(c.w + (size_t)i * c.ldw + n);
                }
#pragma unroll
                for (int j = 0; j < NT; ++j) {
                    if (j0 + j >= taps - 1) continue;
                    if (fresh) v[j] = make_float4(0, 0, 0, 0);
                    y = fma4(w[j], v[j], y);
                    if (j0 + j > 0) *(float4 *)(held + (size_t)(j0 + j - 1) * W4 + n) = v[j];
                }
            }
            if (taps > 1) *(float4 *)(held + (size_t)(taps - 2) * W4 + n) = r;
        }
        store_h4<E>(h + n, y);  // (columns past W: zeros)
    }
}

// ---------------------------------------------------------------- the convolution over longer runs
// TAPS: taps at most.  A thread owns four columns and walks CONV_ROWS rows of one run with the last inputs in registers; the run's first tile carries the state.
template <class E, int TAPS>
__global__ void __launch_bounds__(256) k_conv(const ConvArgs a, const typename E::type *hc, typename E::type *h, int ldh, int W) {
    const int n = (blockIdx.x * 256 + threadIdx.x) * 4, W4 = (W + 3) & ~3, taps = a.taps;
    const RowChunk c = row_chunk(a.runs, a.n_runs, blockIdx.y, CONV_ROWS);
    if (c.n <= 0 || n >= W) return;
    const int run0 = c.row0 - c.pos;
    const bool fresh = a.pos[run0] == 0;
    float *held = taps > 1 ? conv_state(a, run0) + n : nullptr;
    auto at = [&](int i) -> float4 {  // input i of the run; below zero: what the sequence had before
        if (i >= 0) return load_h4<E>(hc + (size_t)(run0 + i) * ldh + n);
        if (fresh || i < 1 - taps) return make_float4(0, 0, 0, 0);
        return *(const float4 *)(held + (size_t)(taps - 1 + i) * W4);
    };
    float4 w[TAPS], v[TAPS];  // v[TAPS - 1]: the row itself
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
        const int i = j - (TAPS - taps);
        w[j] = i >= 0 ? *(const float4 *)(a.w + (size_t)i * a.ldw + n) : make_float4(0, 0, 0, 0);
        v[j] = j > 0 ? at(c.pos + j - TAPS) : make_float4(0, 0, 0, 0);
    }
    if (c.pos == 0 && taps > 1) {
        const int n_rows = a.runs[c.run].n_rows;
        for (int j = 0; j < taps - 1; ++j) *(float4 *)(held + (size_t)j * W4) = at(n_rows - (taps - 1) + j);  // (an older place is read before it is written)
    }
    constexpr int AHEAD = 8;  // rows in flight
    float4 x[AHEAD];
#pragma unroll
    for (int i = 0; i < CONV_ROWS; ++i) {
        if (i % AHEAD == 0)
#pragma unroll
            for (int k = 0; k < AHEAD; ++k) x[k] = load_h4<E>(hc + (size_t)(c.row0 + min(i + k, c.n - 1)) * ldh + n);
        if (i >= c.n) break;
#pragma unroll
        for (int j = 0; j + 1 < TAPS; ++j) v[j] = v[j + 1];
        v[TAPS - 1] = x[i % AHEAD];
        float4 y = fma4(w[TAPS - 1], v[TAPS - 1], v[TAPS - 1]);
#pragma unroll
        for (int j = 0; j + 1 < TAPS; ++j) y = fma4(w[j], v[j], y);
        store_h4<E>(h + (size_t)(c.row0 + i) * ldh + n, y);
    }
}

__global__ void __launch_bounds__(256) k_stream_sum(const float *x, int ldx, int S, float *out, int W) {
    const size_t m = blockIdx.y;
    const int n = blockIdx.x * 256 + threadIdx.x;
    if (n >= W) return;
    float v = 0.0f;
    for (int s = 0; s < S; ++s) v += x[(m * S + s) * ldx + n];
    out[m * W + n] = v;
}

template <class E, int NS>
void stream_go(const StreamUpdateArgs &a, hipStream_t st) {
    const dim3 grid((unsigned)a.M);
#define SU_GO(T_, Q_) hipLaunchKernelGGL((k_stream_update<E, T_, Q_, NS>), grid, dim3(T_), 0, st, a)
    if (a.W <= 256) SU_GO(64, 1);
    else if (a.W <= 1024) SU_GO(256, 1);
    else if (a.M >= 512 && a.W <= 4096) {  // many rows: fewer, longer-lived workgroups per row
        if (a.W <= 2048) SU_GO(256, 2);
        else SU_GO(256, 4);
    } else if (a.W <= 2048) SU_GO(512, 1);
    else if (a.W <= 4096) SU_GO(1024, 1);
    else if (a.W <= 8192) SU_GO(1024, 2);
    else if (a.W <= 16384) SU_GO(1024, 4);
    else SU_GO(1024, 8);
#undef SU_GO
}
template <class E>
void stream_pick(const StreamUpdateArgs &a, hipStream_t st) {
    if (a.S == 1) stream_go<E, 1>(a, st);
    else if (a.S == 2) stream_go<E, 2>(a, st);
    else if (a.S == 3) stream_go<E, 3>(a, st);
    else if (a.S == 4) stream_go<E, 4>(a, st);
    else if (a.S <= 8) stream_go<E, 8>(a, st);
    else stream_go<E, 16>(a, st);
}

template <class E>
void conv_go(const ConvArgs &a, const void *hc, void *h, int ldh, int W, int tiles, hipStream_t st) {
    typedef typename E::type T;
    const dim3 grid((unsigned)((W + 1023) / 1024), (unsigned)tiles);
#define CONV_GO(T_) hipLaunchKernelGGL((k_conv<E, T_>), grid, dim3(256), 0, st, a, (const T *)hc, (T *)h, ldh, W)
    if (a.taps <= 2) CONV_GO(2);
    else if (a.taps == 3) CONV_GO(3);
    else if (a.taps == 4) CONV_GO(4);
    else if (a.taps <= 8) CONV_GO(8);
    else CONV_GO(16);
#undef CONV_GO
}

}  // namespace

int stream_update_launch(int dtype, const StreamUpdateArgs &a, hipStream_t st) {
    if (a.M <= 0) return PIE_OK;
    PIE_REQUIRE(a.W > 0 && a.W <= ROW_UPDATE_MAX_WIDTH && a.S > 0 && a.S <= STREAMS_MAX, PIE_E_SHAPE, "stream update: widths up to 32768, at most 16 streams");
    PIE_REQUIRE(a.ldx % 4 == 0 && a.ldh % 4 == 0 && (!a.y32 || a.ldy % 4 == 0) && a.ldx >= ((a.W + 3) & ~3) && a.ldh >= ((a.W + 3) & ~3), PIE_E_ALIGN, "stream update: row strides must be multiples of 4");
    PIE_REQUIRE(!a.conv.w || (a.conv.taps > 0 && a.conv.taps <= CONV_MAX_TAPS && (a.conv.taps == 1 || a.conv.state)), PIE_E_SHAPE, "stream update: a convolution of 1 .. 16 taps, with its state");
    PIE_REQUIRE(!a.embed.bigram || a.embed.prev, PIE_E_ARG, "stream update: no place for the previous token");
    if (dtype == PIE_F32) stream_pick<ElemF32>(a, st);
    else stream_pick<ElemBF16>(a, st);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

int conv_tiles(int n_rows) { return (n_rows + CONV_ROWS - 1) / CONV_ROWS; }

int conv_launch(int dtype, const ConvArgs &a, const void *hc, void *h, int ldh, int W, int tiles, hipStream_t st) {
    if (tiles <= 0) return PIE_OK;
    PIE_REQUIRE(a.w && a.taps > 0 && a.taps <= CONV_MAX_TAPS && (a.taps == 1 || a.state) && tiles <= 65535 && ldh % 4 == 0, PIE_E_SHAPE, "convolution: 1 .. 16 taps, with their state");
    if (dtype == PIE_F32) conv_go<ElemF32>(a, hc, h, ldh, W, tiles, st);
    else conv_go<ElemBF16>(a, hc, h, ldh, W, tiles, st);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

int stream_sum_launch(const float *x, int ldx, int S, float *out, int M, int W, hipStream_t st) {
    hipLaunchKernelGGL(k_stream_sum, dim3((unsigned)((W + 255) / 256), (unsigned)M), dim3(256), 0, st, x, ldx, S, out, W);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}
