// layer_stack.hip -- native runtime of the layer-stack models: one pass over a list of layers that may all differ (pie_stack_*, include/pie_hip.h).
//
// A pass is a batch of rows, each with its own sequence and position: whole prompts, portions and single decoded tokens are the same thing here.
// A layer is a mixer and a feed-forward, each between two norms.  Mixers:
//   latent attention      [q | latent down] Linear; q -> latent space per head (beside it the latents' RMS norm and their append to the pages); attention
//                         (latent_attn.hip); latents -> values per head, merging the key splits on the way in (more than a few rows: a launch of its own).
//                         With a query latent: [query latent | latent | rotated key | gate] Linear; norms, key rotation, append; queries out of their latent, rotated
//   attention             [q | k | v | gate] Linear; norms, rotation and page writes; attention over keys and values (page_attn.hip)
//   delta rule            [r | k | v | gate | rate | decay] Linear; recurrence (delta_rule.hip)
//   gated delta rule      [q | k | v | gate | step | decay] Linear; short convolution and recurrence (gated_delta.hip)
//   time mixing           the row and its predecessor mixed five ways, beside the update in front; Linears of the mixes; recurrence (time_mix.hip).  It runs alone or
//                         beside an attention over the same row: then one list of Linears makes both inputs (few rows), and one output projection reads both outputs
//   mLSTM                 [q | k | v | gate | i | f] Linear; recurrence (mlstm.hip); head norm and gate (head_out.hip)
//   minGRU                [z | candidate | gate] Linear; recurrence (mingru.hip)
// and an output projection.  Feed-forwards: dense up (relu^2, xIELU, or a gelu gate and up), down; or experts: gate|up and down over the active experts (and a shared one).
// Norms: element-wise ones ride in the epilogue of the kernel that produces their input (x += post(y), h = next(x)); a norm over the whole row is applied,
// with the same additions, by one launch behind the sublayer (row_update.hip), which also takes the experts' weighted sum.
// A layer may norm the sum instead (x = post(alpha x + y)), and may add, behind its sublayers, a vector of the row's token that the row gates (side input: gate Linear, projection, update).
// Hyper-connections keep several residual streams: one launch behind every sublayer mixes them, takes the next sublayer's input out of them, and norms (and, for a mixer,
// convolves) it (stream_update.hip); the first one starts the streams from the embedding.
// A pass of more rows than the weight-streaming Linear is for (BIG_ROWS; bf16) multiplies through the tiled GEMMs instead (w16_gemm.hpp, grouped by expert
// for mixtures); runs of LONG_RUN rows and more use the attentions' long forms (latents: with keys and values spelled out, window_attn.hip) while the
// shorter runs in front of them keep the short ones.
// Where a table names a token's experts, all layers' row lists are made by one launch in front of the pass; a router's are made behind its logits.
#include <cstring>
#include <algorithm>
#include <new>
#include <vector>

#include "mfma_store.hpp"  // MFMA_ACT_*
#include "route.hpp"
#include "stack_types.hpp"

size_t w16l_workspace_bytes(int M, int N, int K);
int w16l_gemm_launch(int dtype, const void *w16m, const void *x, int ldx, int M, int N, int K, void *y, void *workspace, hipStream_t st, const void *bias,
                     void *swiglu_act, bool *fused, int ldy);
int w16l_act_launch(const void *w16m, const void *x, int ldx, int M, int N, int K, void *y, int ldy, int act, float alpha, float beta, const void *bias, hipStream_t st);
int w16l_grouped_launch(const void *w16m, size_t w_stride, const void *x, int ldx, size_t x_rows, const int *list, const void *tiles, int tm, int block, int tile_rows, int N, int K,
                        void *y, int ldy, int act, float act_alpha, float act_limit, hipStream_t st);

namespace {

constexpr int BIG_ROWS = 64;  // more rows than this take the tiled GEMMs
constexpr int LONG_RUN = 64;  // runs of at least this many rows take the attentions' long forms
constexpr int ROUTE_MIN_ROWS = 6, ROUTE_FEW_ROWS = 64;              // up to this many rows, and router weights that one workgroup reads in a few us: chosen beside the norm
constexpr long ROUTE_FEW_WEIGHTS = 256l << 10;
constexpr int CHUNK_RUN = 8;  // runs of at least this many rows take the recurrences' chunk forms

// rows per tile of the grouped GEMM, and a bound on the number of tiles
__host__ __device__ inline int route_tile_rows(long M, int top, int experts) { return M * top >= 96l * experts ? 128 : 64; }
// (an expert's tiles start at a multiple of route_block(): the grouped GEMM runs that many side by side on one XCD, over the same weights)
// (about as many as an expert has: empty tiles cost a workgroup launch each)
constexpr int ROUTE_BLOCK_MAX = 4;
__host__ __device__ inline int route_block(long M, int top, int experts) { return M * top >= 2l * 128 * experts ? 4 : M * top >= 128l * experts ? 2 : 1; }
__host__ __device__ inline int route_max_tiles(long M, int top, int experts) {
    return ((int)(M * top / route_tile_rows(M, top, experts)) + route_block(M, top, experts) * experts + 3) / 4 * 4;
}

__device__ __forceinline__ void route_row(const RouteLayer &L, int m, int lane, const float (&corr)[ROUTE_KEPT]) {
    route_pick(L, L.logits + (size_t)m * L.ld_logits, lane, corr, [&](int k, int e, float w) {
        if (lane == 0) L.chosen[(size_t)m * L.top + k] = e, L.weight[(size_t)m * L.top + k] = w;
    });
}
__global__ void __launch_bounds__(256) k_route_pick(const RouteLayer *layers, int M) {
    const int m = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    const RouteLayer L = layers[0];
    if (m >= M) return;
    float corr[ROUTE_KEPT];
    route_corrections(L, lane, corr);
    route_row(L, m, lane, corr);
}

// the row lists of layers[blockIdx.x]; pick: its router's choice is made here too (few rows: no tiles)
__global__ void __launch_bounds__(1024) k_route(const RouteLayer *layers, const int *ids, int M, int vocab, bool pick) {
    extern __shared__ int s_cnt[];  // [experts] counts, then [experts] cursors
    const RouteLayer L = layers[blockIdx.x];
    if (pick) {
        const int lane = threadIdx.x & 63;
        float corr[ROUTE_KEPT];
        route_corrections(L, lane, corr);
        if (M == 1 && L.top <= 64) {
            if (threadIdx.x < 64) route_single(L, L.logits, lane, corr);
            return;
        }
        for (int m = threadIdx.x >> 6; m < M; m += 16) route_row(L, m, lane, corr);
        __syncthreads();
    }
    const int tr = route_tile_rows(M, L.top, L.experts), rb = route_block(M, L.top, L.experts);
    route_lists(
        L, M, s_cnt,
        [&](int i) {
            if (!L.table) return L.chosen[i];
            return L.table[(size_t)min(max(ids[i / L.top], 0), vocab - 1) * L.top + i % L.top];
        },
        tr, rb, pick ? 0 : route_max_tiles(M, L.top, L.experts));
}

template <class E>
__device__ __forceinline__ void store4(typename E::type *p, float4 y) {
    if constexpr (sizeof(typename E::type) == 2) *(uint2 *)p = make_uint2(pack2<BF16>(y.x, y.y), pack2<BF16>(y.z, y.w));
    else *(float4 *)p = y;
}
template <class E>
__global__ void __launch_bounds__(256) k_stack_embed(const int *ids, const u16 *table, int vocab, int W, float scale, const u16 *positions, int max_positions, const int *pos, bool plain, PointNorm next,
                                                     float *x, int ldx, typename E::type *h, int ldh) {  // plain: h = x; positions: nullable
    const size_t m = blockIdx.y;
    const int n = (blockIdx.x * 256 + threadIdx.x) * 4;
    if (n >= W) return;
    const u16 *src = table + (size_t)min(max(ids[m], 0), vocab - 1) * W + n, *at = positions ? positions + (size_t)min(max(pos[m], 0), max_positions - 1) * W + n : nullptr;
    if (n + 4 <= W && !(W & 3)) {
        const uint2 t = *(const uint2 *)src;
        float4 v = make_float4(lo_f32<BF16>(t.x) * scale, hi_f32<BF16>(t.x) * scale, lo_f32<BF16>(t.y) * scale, hi_f32<BF16>(t.y) * scale);
        if (at) {
            const uint2 p = *(const uint2 *)at;
            v.x += lo_f32<BF16>(p.x), v.y += hi_f32<BF16>(p.x), v.z += lo_f32<BF16>(p.y), v.w += hi_f32<BF16>(p.y);
        }
        const float4 y = plain ? v : point_norm4(next, n, v);
        *(float4 *)(x + m * ldx + n) = v;
        store4<E>(h + m * ldh + n, y);
        return;
    }
    for (int i = 0; i < min(4, W - n); ++i) {
        const float v = BF16::to_f32(src[i]) * scale + (at ? BF16::to_f32(at[i]) : 0.0f);
        x[m * ldx + n + i] = v;
        h[m * ldh + n + i] = E::pack(plain ? v : point_norm(next, n + i, v));
    }
}

// y = gelu(y) * the row's token's side vector (bf16, many rows)
__global__ void __launch_bounds__(256) k_side_gate(u16 *y, int ldy, TokenVectors side, int M, int N) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x, m = i / N, n = i % N;
    if (m >= (size_t)M) return;
    u16 *p = y + m * ldy + n;
    *p = BF16::from_f32(gelu_tanh<false>(BF16::to_f32(*p)) * BF16::to_f32(token_vector(side, m)[n]));
}

// y = sum over the token's slots of its experts' weighted outputs (+ sigmoid(gate . input) * shared output); x += post(y); h = next(x)
struct CombineArgs {
    const void *part, *part_s;   // [M * top][ldp] by position, [M][ldp_s]
    int ldp, ldp_s;
    const int *place;
    const float *weight;         // [M * top] or nullptr: 1 / top each
    int top, W;
    const float *gate;           // [W] or nullptr
    PointNorm pre, post, next;   // pre: the sublayer's input norm (the gate's dot product is taken in fp32 on it)
    float *x;
    int ldx;
    void *h;
    int ldh;
};
template <class P>
__device__ __forceinline__ float4 load4(const void *p, size_t i) {
    if constexpr (sizeof(typename P::type) == 4) return *(const float4 *)((const float *)p + i);
    else {
        const uint2 v = *(const uint2 *)((const u16 *)p + i);
        return make_float4(lo_f32<BF16>(v.x), hi_f32<BF16>(v.x), lo_f32<BF16>(v.y), hi_f32<BF16>(v.y));
    }
}
template <class E, class P>  // P: element type of the experts' outputs.  One workgroup per row, four columns per thread and pass.
__global__ void __launch_bounds__(1024) k_moe_combine(const CombineArgs a) {
    __shared__ float red[16];
    const size_t m = blockIdx.x;
    float *x = a.x + m * a.ldx;
    constexpr int U = 8;  // slots in flight
    float4 v[U], vs = make_float4(0, 0, 0, 0), xv = vs;
    int n = threadIdx.x * 4;
    float share[U];
    auto fetch = [&](int s0) {
#pragma unroll
        for (int u = 0; u < U; ++u)
            if (s0 + u < a.top) share[u] = a.weight ? a.weight[m * a.top + s0 + u] : 1.0f / (float)a.top, v[u] = load4<P>(a.part, (size_t)a.place[m * a.top + s0 + u] * a.ldp + n);
    };
    auto fetch_row = [&] {  // (rows of x, part and the norms' paddings: a quad that starts inside W is readable up to the next multiple of 4)
        fetch(0);
        if (a.gate) vs = load4<P>(a.part_s, m * a.ldp_s + n);
        xv = *(const float4 *)(x + n);
    };
    if (n < a.W) fetch_row();
    float g = 0.0f;
    if (a.gate) {
        float d = 0.0f;
        for (int k = n; k < a.W; k += blockDim.x * 4) {
            const float4 q = point_norm4(a.pre, k, k == n ? xv : *(const float4 *)(x + k)), w = *(const float4 *)(a.gate + k);
            d += (fmaf(q.x, w.x, q.y * w.y) + fmaf(q.z, w.z, q.w * w.w));  // (columns past W: zero gate weights)
        }
        d = wave_sum(d);
        if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = d;
        __syncthreads();
        d = red[0];
        for (int i = 1; i < (int)blockDim.x / 64; ++i) d += red[i];
        g = 1.0f / (1.0f + expf(-d));
    }
    for (; n < a.W; n += blockDim.x * 4) {
        if (n != (int)threadIdx.x * 4) fetch_row();
        float y[4] = {0, 0, 0, 0};
        for (int s0 = 0; s0 < a.top; s0 += U) {
            if (s0) fetch(s0);
#pragma unroll
            for (int u = 0; u < U; ++u)
                if (s0 + u < a.top) y[0] = fmaf(share[u], v[u].x, y[0]), y[1] = fmaf(share[u], v[u].y, y[1]), y[2] = fmaf(share[u], v[u].z, y[2]), y[3] = fmaf(share[u], v[u].w, y[3]);
        }
        if (a.gate) y[0] = fmaf(g, vs.x, y[0]), y[1] = fmaf(g, vs.y, y[1]), y[2] = fmaf(g, vs.z, y[2]), y[3] = fmaf(g, vs.w, y[3]);
        const float4 q = point_norm4(a.post, n, make_float4(y[0], y[1], y[2], y[3]));
        const float4 r = make_float4(xv.x + q.x, xv.y + q.y, xv.z + q.z, xv.w + q.w), hn = point_norm4(a.next, n, r);
        typename E::type *h = (typename E::type *)a.h + m * a.ldh + n;
        if (n + 4 <= a.W) {
            *(float4 *)(x + n) = r;
            store4<E>(h, hn);
        } else {
            const float re[4] = {r.x, r.y, r.z, r.w}, he[4] = {hn.x, hn.y, hn.z, hn.w};
            for (int i = 0; i < a.W - n; ++i) x[n + i] = re[i], h[i] = E::pack(he[i]);
        }
    }
}

// x += post(y); h = next(x), four columns per thread (y, h: bf16)
__global__ void __launch_bounds__(256) k_point_residual(const u16 *y, int ldy, PointNorm post, PointNorm next, float *x, int ldx, u16 *h, int ldh, int W) {
    const size_t m = blockIdx.y;
    const int n = (blockIdx.x * 256 + threadIdx.x) * 4;
    if (n >= W) return;
    if (n + 4 <= W && !(ldy & 3)) {
        const uint2 yv = *(const uint2 *)(y + m * ldy + n);
        float4 *xp = (float4 *)(x + m * ldx + n), v = *xp;
        const float4 q = point_norm4(post, n, make_float4(lo_f32<BF16>(yv.x), hi_f32<BF16>(yv.x), lo_f32<BF16>(yv.y), hi_f32<BF16>(yv.y)));
        v.x += q.x, v.y += q.y, v.z += q.z, v.w += q.w;
        *xp = v;
        store4<ElemBF16>(h + m * ldh + n, point_norm4(next, n, v));
        return;
    }
    for (int i = n; i < min(n + 4, W); ++i) {
        const float v = x[m * ldx + i] + point_norm(post, i, BF16::to_f32(y[m * ldy + i]));
        x[m * ldx + i] = v;
        h[m * ldh + i] = BF16::from_f32(point_norm(next, i, v));
    }
}

// log-softmax and greedy token over fp32 logits: per-tile (max, sum, first argmax), then every workgroup of a row merges the row's tiles
constexpr int ST_TILES = 64;
struct RowStat {
    float max, sum;
    int arg, pad;
};
__global__ void __launch_bounds__(256) k_f32_stats(const float *logits, int V, RowStat *stats) {
    __shared__ float s_max[4], s_sum[4];
    __shared__ int s_arg[4];
    logits += (size_t)blockIdx.y * V;
    const int len = (V + ST_TILES - 1) / ST_TILES, begin = blockIdx.x * len, end = min(V, begin + len), wave = threadIdx.x >> 6;
    float mx = -INFINITY;
    int arg = 0x7fffffff;
    for (int i = begin + threadIdx.x; i < end; i += 256)
        if (logits[i] > mx) mx = logits[i], arg = i;
    const float wm = wave_max(mx);
    int cand = mx == wm ? arg : 0x7fffffff;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) cand = min(cand, __shfl_xor(cand, o, 64));
    if ((threadIdx.x & 63) == 0) s_max[wave] = wm, s_arg[wave] = cand;
    __syncthreads();
    float tm = s_max[0];
    int ta = s_arg[0];
    for (int w = 1; w < 4; ++w)
        if (s_max[w] > tm || (s_max[w] == tm && s_arg[w] < ta)) tm = s_max[w], ta = s_arg[w];
    float se = 0.0f;
    for (int i = begin + threadIdx.x; i < end; i += 256) se += expf(logits[i] - tm);
    se = wave_sum(se);
    if ((threadIdx.x & 63) == 0) s_sum[wave] = se;
    __syncthreads();
    if (threadIdx.x == 0) stats[blockIdx.y * ST_TILES + blockIdx.x] = {tm, (s_sum[0] + s_sum[1]) + (s_sum[2] + s_sum[3]), ta, 0};
}
__global__ void __launch_bounds__(256) k_f32_finish(const float *logits, int V, const RowStat *stats, float *logprobs, int *next, int advance, int *ids, int *pos,
                                                    int *history, int history_len) {
    const size_t r = blockIdx.y;
    const int lane = threadIdx.x & 63;
    const RowStat st = stats[r * ST_TILES + lane];  // (every wave merges the same 64 tiles)
    const float mx = wave_max(st.max);
    int cand = st.max == mx ? st.arg : 0x7fffffff;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) cand = min(cand, __shfl_xor(cand, o, 64));
    const float lse = mx + logf(wave_sum(st.sum > 0.0f ? st.sum * expf(st.max - mx) : 0.0f));
    if (logprobs)
        for (int i = blockIdx.x * 256 + threadIdx.x; i < V; i += gridDim.x * 256) logprobs[r * V + i] = logits[r * V + i] - lse;
    if (blockIdx.x == 0 && threadIdx.x == 0) {
        next[r] = cand;
        if (advance) {
            const int p = pos[r] + 1;
            ids[r] = cand, pos[r] = p;
            if (history && r == 0 && p < history_len) history[p] = cand;
        }
    }
}

template <class T>
struct Buf {  // a device buffer that only grows; new memory is zero (row paddings stay finite), with slack for a read past the last row's end
    static constexpr size_t SLACK = 1024;  // elements (bytes for char)
    T *p = nullptr;
    size_t cap = 0;
    int need(size_t n, bool *moved) {
        if (n <= cap) return PIE_OK;
        if (p) PIE_HIP_TRY(hipFree(p));
        p = nullptr, cap = 0;
        PIE_HIP_TRY(hipMalloc((void **)&p, (n + SLACK) * sizeof(T)));
        PIE_HIP_TRY(hipMemset(p, 0, (n + SLACK) * sizeof(T)));
        cap = n, *moved = true;
        return PIE_OK;
    }
    ~Buf() {
        if (p) (void)hipFree(p);
    }
};

int up8(int n) { return (n + 7) & ~7; }
int up64(int n) { return (n + 63) & ~63; }

struct GraphKey {
    pie_stack_batch b;
    std::vector<void *> slabs;
    std::vector<float *> states;
    std::vector<int32_t> runs;
    bool same(const GraphKey &o) const { return memcmp(&b, &o.b, sizeof b) == 0 && slabs == o.slabs && states == o.states && runs == o.runs; }
};
struct GraphSlot {
    GraphKey key;
    hipGraphExec_t exec = nullptr;
    unsigned long long used = 0;
};

}  // namespace

struct pie_stack {
    pie_stack_config cfg;
    std::vector<pie_stack_layer> layers;
    std::vector<char> have;
    // workspace, by rows of a pass
    Buf<float> x, c_raw, part, part_s, attn_ws, gemm_ws, y32, logits_e, rec_ws, rec_o, rec_den;
    Buf<char> h, hc, q, qu, cq, ql, oc, o, act, act_e, act_s, y, ctx, kv, mixes, mixed, side;
    Buf<RowStat> stats;
    Buf<int> route_ints;
    Buf<RouteLayer> route_dev;
    Buf<int> arrived;               // rows that have chosen their experts (zero between launches)
    std::vector<RouteLayer> route;  // per layer; experts == 0: not a mixture
    int route_rows = 0, n_table = 0, route_lds = 0;  // n_table: mixtures whose experts a table names (in front in route_dev)
    std::vector<int> route_at;      // layer -> entry of route_dev
    std::vector<GraphSlot> graphs;
    unsigned long long tick = 0;
    int launches = 0;
    void drop_graphs() {
        for (GraphSlot &g : graphs)
            if (g.exec) (void)hipGraphExecDestroy(g.exec);
        graphs.clear();
    }
    ~pie_stack() { drop_graphs(); }
};

namespace {

size_t esize(const pie_stack *s) { return s->cfg.dtype == PIE_F32 ? 4 : 2; }
bool pointwise(const pie_stack_norm &n) { return n.kind == PIE_NORM_DYN_TANH; }
PointNorm norm_of(const pie_stack_norm &n) { return {n.w, n.b, n.param}; }
StackNorm row_norm_of(const pie_stack_norm &n) { return {n.w, n.b, n.param, n.kind}; }
bool is_moe(const pie_stack_layer &L) { return L.ff == PIE_FF_TABLE_MOE || L.ff == PIE_FF_ROUTED_MOE; }
KvGeometry geometry(const pie_stack_layer &L) { return kv_geometry(L.heads, L.kv_heads, L.dim, L.vdim); }
bool is_dense(const pie_stack_layer &L) { return L.ff == PIE_FF_RELU2 || L.ff == PIE_FF_XIELU || L.ff == PIE_FF_GEGLU; }
bool has_time_mix(const pie_stack_layer &L) { return L.time_mix.heads > 0; }
int gated_channels(const pie_stack_layer &L);
bool own_cache(const pie_stack_layer &L) { return (L.mixer == PIE_MIXER_LATENT && (!L.q_rank || L.kv_from < 0)) || (L.mixer == PIE_MIXER_ATTENTION && L.kv_from < 0); }
// columns of the mixer's input projection, and what its output projection reads
int in_columns(const pie_stack_layer &L) {
    const int gate = L.out_gate ? up8(L.heads) : 0;
    switch (L.mixer) {
        case PIE_MIXER_LATENT:
            if (L.q_rank) return up8(L.q_rank) + (own_cache(L) ? up8(L.rank) + up8(L.rot_dim) : 0) + gate;
            return L.heads * up8(L.dim) + up8(L.rank);
        case PIE_MIXER_DELTA: return 5 * L.heads * up8(L.dim) + up8(L.rank);
        case PIE_MIXER_MLSTM: return 2 * L.heads * (up8(L.dim) + up8(L.vdim)) + 2 * up8(L.heads);
        case PIE_MIXER_MINGRU: return 3 * up8(L.dim);
        case PIE_MIXER_GATED_DELTA: return gated_channels(L) + L.heads * up8(L.vdim) + 2 * up8(L.heads);
        case PIE_MIXER_TIME_MIX: return 0;
        default: return L.heads * up8(L.dim) + (own_cache(L) ? L.kv_heads * (up8(L.dim) + (L.row_norm ? 0 : up8(L.vdim))) : 0) + gate;
    }
}
int time_mix_columns(const pie_stack_layer &L) { return has_time_mix(L) ? L.time_mix.heads * up8(L.time_mix.dim) : 0; }  // of each of its projections, and of its output
int out_columns(const pie_stack_layer &L) {
    if (L.mixer == PIE_MIXER_TIME_MIX) return time_mix_columns(L);
    return L.heads * up8(L.mixer == PIE_MIXER_DELTA || L.mixer == PIE_MIXER_MINGRU ? L.dim : L.vdim) + time_mix_columns(L);
}
int gated_channels(const pie_stack_layer &L) { return gated_delta_channels(L.heads, L.kv_heads, up8(L.dim), up8(L.vdim)); }
int up4(int n) { return (n + 3) & ~3; }
int latent_row(const pie_stack_layer &L) { return up8(L.rank) + up8(L.rot_dim); }  // numbers of a cached latent row

// A layer's recurrent state: the mixer's (a gated delta rule's with its convolution's last inputs at `ring`), the last inputs of the convolution in front of it, (layer 0) the embedding's
// previous token, and the previous row that time mixing reads
struct StateLayout {
    size_t conv, prev, total;  // where the second and the third begin
    size_t ring, row;
};
StateLayout state_layout(const pie_stack *s, int i) {
    const pie_stack_layer &L = s->layers[i];
    size_t mixer = 0;
    if (L.mixer == PIE_MIXER_DELTA) mixer = (size_t)L.heads * L.dim * L.dim;
    else if (L.mixer == PIE_MIXER_MLSTM) mixer = mlstm_state_floats(L.heads, L.dim, L.vdim);
    else if (L.mixer == PIE_MIXER_MINGRU) mixer = L.dim;
    else if (has_time_mix(L)) mixer = (size_t)L.time_mix.heads * L.time_mix.dim * L.time_mix.dim;
    size_t ring = 0;
    if (L.mixer == PIE_MIXER_GATED_DELTA) {
        ring = ((size_t)L.heads * L.dim * L.vdim + 3) / 4 * 4;
        mixer = ring + (L.mix_taps > 1 ? (size_t)L.mix_taps * gated_channels(L) : 0);
    }
    const size_t row = has_time_mix(L) ? up4(s->cfg.width) : 0, conv = L.conv_taps > 1 ? (size_t)(L.conv_taps - 1) * up4(s->cfg.width) : 0, prev = i == 0 && s->cfg.bigram ? 4 : 0;
    if (!conv && !prev && (L.mixer == PIE_MIXER_DELTA || !mixer)) return {mixer, mixer, mixer, 0, 0};
    mixer = (mixer + 3) / 4 * 4;
    return {mixer, mixer + conv, mixer + conv + prev + row, ring, mixer + conv + prev};
}

// How a pass is laid out: rows of the leading short runs, and what the long runs behind them see.
struct Plan {
    bool big;
    int short_rows, short_runs, long_rows;
};
Plan plan_pass(const pie_stack *s, const pie_stack_batch &b) {
    Plan p = {s->cfg.dtype == PIE_BF16 && b.n_rows > BIG_ROWS, 0, 0, 0};
    while (p.short_runs < b.n_runs && (!p.big || b.runs_host[4 * p.short_runs + 1] < LONG_RUN)) p.short_rows += b.runs_host[4 * p.short_runs++ + 1];
    p.long_rows = b.n_rows - p.short_rows;
    return p;
}
bool spelled_out(const pie_stack_layer &L) { return L.w_kv && up8(L.dim) + up8(L.rot_dim) <= WINDOW_ATTN_MAX_DIM && up8(L.vdim) <= WINDOW_ATTN_MAX_DIM; }
// tokens the long runs of a layer see
size_t plan_context(const pie_stack_batch &b, const Plan &p, int window) {
    size_t n = 0;
    for (int i = p.short_runs; i < b.n_runs; ++i) {
        const int32_t *r = b.runs_host + 4 * i;
        const int first = window > 0 ? std::max(0, r[3] - window + 1) : 0;
        n += r[3] + r[1] - first;
    }
    return n;
}

// the leading runs that take a recurrence's step form, their rows, and the chunks of those behind them
struct ChunkPart {
    int runs, rows, chunks;
};
bool chunk_form(const pie_stack *s, const pie_stack_layer &L) { return L.mixer != PIE_MIXER_MLSTM || (s->cfg.dtype == PIE_BF16 && L.dim <= MLSTM_CHUNK_MAX_DIM); }
ChunkPart chunk_part(const pie_stack *s, const pie_stack_batch &b, const pie_stack_layer &L) {
    ChunkPart p = {0, 0, 0};
    const bool chunks = chunk_form(s, L);
    while (p.runs < b.n_runs && (!chunks || b.runs_host[4 * p.runs + 1] < CHUNK_RUN)) p.rows += b.runs_host[4 * p.runs++ + 1];
    for (int i = p.runs; i < b.n_runs; ++i) {
        const int n = b.runs_host[4 * i + 1];
        p.chunks += L.mixer == PIE_MIXER_MLSTM ? mlstm_chunks(n) : L.mixer == PIE_MIXER_MINGRU ? mingru_chunks(n) : delta_chunks(n);
    }
    return p;
}

int stack_reserve(pie_stack *s, const pie_stack_batch &b, const Plan &plan, hipStream_t st) {
    const size_t M = (size_t)b.n_rows, E = esize(s), W64 = up64(s->cfg.width), WA = act_stride(s->cfg.width);
    size_t mx = 0, md = 0, sd = 0, q = 0, c = 0, ql = 0, o = 0, act = 0, act_e = 0, act_s = 0, part = 0, part_s = 0, ints = 0, ctx = 0, kv = 0, ws = 0, le = 0, rw = 0, ro = 0, rd = 0, hc = 0, qu = 0, cq = 0;
    const size_t streams = std::max(s->cfg.streams, 1);
    auto gemm = [&](int N, int K) { ws = std::max(ws, w16l_workspace_bytes((int)M, N, K) / 4); };
    for (const pie_stack_layer &L : s->layers) {
        const int NI = in_columns(L), KO = out_columns(L);
        q = std::max(q, (size_t)NI), o = std::max(o, (size_t)act_stride(KO));
        if (plan.big && NI) gemm(NI, s->cfg.width);
        if (plan.big) gemm(s->cfg.width, KO);
        if (L.mixer == PIE_MIXER_LATENT) {
            c = std::max(c, (size_t)up8(L.rank)), ql = std::max(ql, (size_t)L.heads * up8(L.rank));
            if (L.q_rank) {
                const int NQ = L.heads * (up8(L.dim) + up8(L.rot_dim));
                qu = std::max(qu, (size_t)NQ), cq = std::max(cq, (size_t)act_stride(L.q_rank));
                if (plan.big) gemm(NQ, L.q_rank);
            } else if (plan.big) gemm(L.heads * up8(L.dim), s->cfg.width), gemm(up8(L.rank), s->cfg.width);
            if (plan.long_rows && spelled_out(L)) {
                const size_t n = plan_context(b, plan, L.window), nkv = L.heads * (up8(L.dim) + up8(L.vdim));
                ctx = std::max(ctx, n * act_stride(latent_row(L))), kv = std::max(kv, n * nkv);
                ws = std::max(ws, w16l_workspace_bytes((int)n, (int)nkv, L.rank) / 4);
            }
        }
        if (L.conv_taps > 0 && b.n_runs < b.n_rows) hc = WA;
        if (L.mixer == PIE_MIXER_GATED_DELTA) {
            const int chunks = chunk_part(s, b, L).chunks;
            md = std::max(md, (size_t)gated_channels(L)), ro = std::max(ro, (size_t)L.heads * up8(L.vdim));
            if (chunks) rw = std::max(rw, gated_delta_ws_floats(chunks, L.heads, L.dim));
        }
        if (has_time_mix(L)) {
            const int chunks = chunk_part(s, b, L).chunks, NT = time_mix_columns(L), R8 = up8(L.time_mix.rank);
            mx = TIME_MIXES * WA, md = std::max(md, (size_t)4 * NT + R8), ro = std::max(ro, (size_t)NT);
            if (chunks) rw = std::max(rw, time_mix_ws_floats(chunks, L.time_mix.heads, L.time_mix.dim));
            if (plan.big) gemm(NT, s->cfg.width), gemm(R8, s->cfg.width);
        }
        if (L.w_side_gate) {
            sd = act_stride(s->cfg.side_dim);
            if (plan.big) gemm(up8(s->cfg.side_dim), s->cfg.width), gemm(s->cfg.width, s->cfg.side_dim);
        }
        if (L.mixer == PIE_MIXER_MLSTM) ro = std::max(ro, (size_t)L.heads * up8(L.vdim)), rd = std::max(rd, (size_t)L.heads);
        if (L.mixer == PIE_MIXER_DELTA || L.mixer == PIE_MIXER_MLSTM || L.mixer == PIE_MIXER_MINGRU) {
            const int chunks = chunk_part(s, b, L).chunks;
            if (chunks && L.mixer == PIE_MIXER_DELTA) rw = std::max(rw, delta_ws_floats(chunks, L.heads, L.dim)), ro = std::max(ro, (size_t)L.heads * up8(L.dim));
            else if (chunks && L.mixer == PIE_MIXER_MLSTM) rw = std::max(rw, mlstm_ws_floats(chunks, L.heads, L.dim, L.vdim));
            else if (chunks) rw = std::max(rw, mingru_ws_floats(chunks, L.dim));
        }
        if (is_dense(L)) {
            act = std::max(act, (size_t)act_stride(L.ff_size));
            if (plan.big) gemm(s->cfg.width, L.ff_size);
        }
        if (is_moe(L)) {
            act_e = std::max(act_e, (size_t)L.top * act_stride(L.ff_size)), part = std::max(part, (size_t)L.top * W64);
            if (L.ff == PIE_FF_ROUTED_MOE) le = std::max(le, (size_t)up8(L.experts));
            if (L.shared_size) {
                act_s = std::max(act_s, (size_t)act_stride(L.shared_size)), part_s = W64;
                if (plan.big) gemm(s->cfg.width, L.shared_size);
            }
        }
    }
    bool moved = false;
    int rc = 0;
    if ((rc = s->x.need(M * streams * W64, &moved)) || (rc = s->c_raw.need(M * c, &moved)) || (rc = s->part.need(M * part, &moved)) || (rc = s->part_s.need(M * part_s, &moved)) ||
        (rc = s->h.need(M * WA * E, &moved)) || (rc = s->q.need(M * q * E, &moved)) || (rc = s->ql.need(M * ql * E, &moved)) || (rc = s->oc.need(M * ql * E, &moved)) ||
        (rc = s->o.need(M * o * E, &moved)) || (rc = s->act.need(M * act * E, &moved)) || (rc = s->act_e.need(M * act_e * E, &moved)) ||
        (rc = s->act_s.need(M * act_s * E, &moved)) || (rc = s->stats.need((size_t)b.n_want * ST_TILES, &moved)) || (rc = s->y.need(plan.big ? M * W64 * E : 0, &moved)) ||
        (rc = s->y32.need(plan.big ? 0 : M * W64, &moved)) || (rc = s->logits_e.need(M * le, &moved)) || (rc = s->rec_ws.need(rw, &moved)) || (rc = s->rec_o.need(M * ro, &moved)) ||
        (rc = s->rec_den.need(M * rd, &moved)) || (rc = s->hc.need(M * hc * E, &moved)) || (rc = s->mixes.need(M * mx * E, &moved)) || (rc = s->mixed.need(M * md * E, &moved)) || (rc = s->side.need(M * sd * E, &moved)) || (rc = s->qu.need(M * qu * E, &moved)) || (rc = s->cq.need(M * cq * E, &moved)) || (rc = s->ctx.need(ctx * E, &moved)) ||
        (rc = s->kv.need(kv * E, &moved)) || (rc = s->gemm_ws.need(ws, &moved)))
        return rc;
    int n_moe = 0;
    s->n_table = 0;
    for (const pie_stack_layer &L : s->layers) n_moe += is_moe(L), s->n_table += L.ff == PIE_FF_TABLE_MOE;
    if (n_moe && ((int)M > s->route_rows || moved)) {
        s->route_rows = std::max(s->route_rows, (int)M);
        const size_t R = (size_t)s->route_rows;
        // (at most this many tiles for any pass of up to R rows: 64-row tiles and one ragged block of tiles per expert)
        auto tiles = [&](const RouteLayer &r) { return (R * r.top / 64 + ROUTE_BLOCK_MAX * r.experts + 3) / 4 * 4; };
        auto lists = [&](const RouteLayer &r) { return (2 * (size_t)r.experts + 1 + 2 * R * r.top + (r.table ? 0 : 2 * R * r.top) + 3) / 4 * 4; };
        for (const RouteLayer &r : s->route)
            if (r.experts) ints += lists(r) + 4 * tiles(r);
        if ((rc = s->route_ints.need(ints, &moved)) || (rc = s->route_dev.need(n_moe, &moved)) || (rc = s->arrived.need(1, &moved))) return rc;
        int *p = s->route_ints.p, at[2] = {0, s->n_table};
        std::vector<RouteLayer> dev(n_moe);
        s->route_lds = 0, s->route_at.assign(s->layers.size(), 0);
        for (size_t i = 0; i < s->layers.size(); ++i) {
            RouteLayer &r = s->route[i];
            if (!r.experts) continue;
            r.tiles = (int4 *)p, p += 4 * tiles(r);
            r.active = p, r.offset = r.active + r.experts, r.list = r.offset + r.experts + 1, r.place = r.list + R * r.top;
            if (!r.table) r.chosen = r.place + R * r.top, r.weight = (float *)(r.chosen + R * r.top), r.logits = s->logits_e.p, r.ld_logits = up8(r.experts);
            p += lists(r);
            r.max_active = r.experts;
            s->route_lds = std::max(s->route_lds, 2 * r.experts * 4);
            dev[s->route_at[i] = at[r.table ? 0 : 1]++] = r;
        }
        PIE_HIP_TRY(hipStreamSynchronize(st));
        PIE_HIP_TRY(hipMemcpy(s->route_dev.p, dev.data(), dev.size() * sizeof(RouteLayer), hipMemcpyHostToDevice));
        moved = true;
    }
    if (moved) {
        PIE_HIP_TRY(hipDeviceSynchronize());
        s->drop_graphs();
    }
    return PIE_OK;
}

// key splits of a layer's attention: enough workgroups for the chip, at least 64 keys each; from capacities only, so that a captured step keeps its plan
int plan_splits(const pie_stack_batch &b, const pie_stack_layer &L, int n_tiles) {
    if (n_tiles <= 0) return 1;
    long ctx = (long)b.table_width * PAGE_TOKENS;
    if (L.window > 0 && L.window + 64 < ctx) ctx = L.window + 64;
    if (L.chunk > 0 && L.chunk + 64 < ctx) ctx = L.chunk + 64;
    long s = 256 / n_tiles;
    s = std::min(s, ctx / 64);
    s = std::min(s, 64L);
    return (int)std::max(s, 1L);
}

// the rows and runs of a pass that take a layer's short attention form, and their tiles
struct ShortPart {
    int M, runs, tiles;
};
ShortPart short_part(const pie_stack *s, const pie_stack_batch &b, const Plan &plan, const pie_stack_layer &L) {
    const bool attn = L.mixer == PIE_MIXER_ATTENTION, split = plan.long_rows && (attn ? page_attn_mfma(s->cfg.dtype, geometry(L)) : spelled_out(L));
    ShortPart p = {split ? plan.short_rows : b.n_rows, split ? plan.short_runs : b.n_runs, 0};
    for (int i = 0; i < p.runs; ++i) p.tiles += attn ? page_attn_tiles(b.runs_host[4 * i + 1], geometry(L)) : latent_attn_tiles(b.runs_host[4 * i + 1], L.heads);
    return p;
}
// floats of key-split workspace a layer's attention needs
size_t attn_ws(const pie_stack *s, const pie_stack_batch &b, const Plan &plan, const pie_stack_layer &L) {
    if (L.mixer != PIE_MIXER_LATENT && L.mixer != PIE_MIXER_ATTENTION) return 0;
    const ShortPart p = short_part(s, b, plan, L);
    if (!p.tiles) return 0;
    const int splits = plan_splits(b, L, p.tiles);
    return L.mixer == PIE_MIXER_ATTENTION ? page_attn_ws_floats(p.M, geometry(L), splits) : latent_attn_ws_floats(p.M, L.heads, L.rank, splits);
}

// what a sublayer's input is made of: the norm in front of it, with hyper-connections the streams' shares (nullptr: their sum), the layer whose convolution follows (or -1), and the layer
// whose time mixing reads it (or -1)
struct Into {
    const pie_stack_norm *norm;
    const float *in;
    int conv, mix;
};
// what a sublayer's output goes through on its way into the residual: x += norm(y + bias), or (after) x = norm(scale x + y + bias)
struct OutOf {
    const pie_stack_norm &norm;
    const float *hyper;  // hyper-connections: the sublayer's, instead
    const u16 *bias;
    bool after;
    float scale;
};
OutOf out_of(const pie_stack_layer &L, const pie_stack_norm &norm, const float *hyper, const void *bias) { return {norm, hyper, (const u16 *)bias, L.norm_after != 0, L.residual_scale}; }

struct Pass {
    pie_stack *s;
    const pie_stack_batch &b;
    Plan plan;
    hipStream_t st;
    int rc = PIE_OK, launches = 0;
    // many rows: y = x . W^T rounded to bf16, or the SwiGLU activation of an interleaved matrix
    void gemm(const void *w, const void *x, int ldx, int M, int N, int K, void *y, int ldy, bool swiglu = false) {
        if (!rc)
            rc = w16l_gemm_launch(PIE_BF16, w, x, ldx, M, N, K, swiglu ? nullptr : y, s->gemm_ws.p, st, nullptr, swiglu ? y : nullptr, nullptr, ldy), ++launches;
    }
    // the slots and runs a layer's state belongs to (at: its place in the state)
    ConvArgs conv_args(int li, size_t at) const {
        ConvArgs c = {};
        c.pos = b.pos, c.row_seq = b.row_seq, c.slots = b.slots, c.n_seqs = b.n_seqs, c.n_slots = (int)b.n_slots, c.runs = (const RowRun *)b.runs, c.n_runs = b.n_runs;
        if (b.states && b.states[li]) c.state = b.states[li] + at, c.slot_floats = state_layout(s, li).total;
        return c;
    }
    // the streams take y = s->y (bf16; many rows) or s->y32 (hyper: the sublayer's connections), or start from the embedding (hyper null); h = the next sublayer's input
    void streams(const float *hyper, const Into &next) {
        if (rc) return;
        const int W = s->cfg.width, WA = act_stride(W), S = s->cfg.streams;
        StreamUpdateArgs a = {};
        a.x = s->x.p, a.ldx = up64(W), a.S = S, a.in = next.in, a.next = row_norm_of(*next.norm), a.ldh = WA, a.M = b.n_rows, a.W = W, a.single = b.n_runs == b.n_rows;
        ConvArgs conv = {};
        if (next.conv >= 0) {
            conv = conv_args(next.conv, state_layout(s, next.conv).conv);
            conv.w = s->layers[next.conv].conv, conv.taps = s->layers[next.conv].conv_taps, conv.ldw = up64(W);
        }
        const bool behind = next.conv >= 0 && !a.single;  // the convolution has its own launch
        if (hyper) {
            a.y = plan.big ? (const void *)s->y.p : s->y32.p, a.y32 = !plan.big, a.ldy = plan.big ? W : up64(W), a.out = hyper + S, a.mix = hyper + 2 * S;
            if (next.conv >= 0) a.conv = conv;
        } else {
            a.conv = next.conv >= 0 ? conv : conv_args(0, 0);
            StackEmbed &e = a.embed;
            e.ids = b.ids, e.table = (const u16 *)s->cfg.embed, e.scale = s->cfg.embed_scale, e.vocab = s->cfg.vocab;
            e.positions = (const u16 *)s->cfg.positions, e.max_positions = s->cfg.max_positions;
            e.bigram = (const u16 *)s->cfg.bigram, e.buckets = s->cfg.buckets, e.mul_prev = s->cfg.mul_prev, e.mul_cur = s->cfg.mul_cur;
            if (e.bigram) e.prev = b.states[0] + state_layout(s, 0).prev;
        }
        a.h = behind ? s->hc.p : s->h.p;
        rc = stream_update_launch(s->cfg.dtype, a, st), ++launches;
        if (rc || !behind) return;
        int tiles = 0;
        for (int i = 0; i < b.n_runs; ++i) tiles += conv_tiles(b.runs_host[4 * i + 1]);
        rc = conv_launch(s->cfg.dtype, conv, s->hc.p, s->h.p, WA, W, tiles, st), ++launches;
    }
    // x += post(y); h = next(x) over y = s->y (bf16; many rows) or s->y32
    // route (few rows): the layer whose experts the rows choose on their way
    TokenMixArgs mix_args(int li) const {
        TokenMixArgs t = {};
        const StateLayout at = state_layout(s, li);
        t.mu = s->layers[li].time_mix.mu, t.ldmu = up64(s->cfg.width), t.state = b.states[li] + at.row, t.slot_floats = at.total;
        t.pos = b.pos, t.row_seq = b.row_seq, t.slots = b.slots, t.n_seqs = b.n_seqs, t.n_slots = (int)b.n_slots, t.runs = (const RowRun *)b.runs, t.n_runs = b.n_runs;
        t.out = s->mixes.p, t.ldo = act_stride(s->cfg.width);
        return t;
    }
    // the mixes that layer li's time mixing reads, of the residual as it stands
    void token_mix(int li) {
        if (!rc) rc = token_mix_launch(s->cfg.dtype, mix_args(li), s->x.p, up64(s->cfg.width), b.n_rows, s->cfg.width, st), ++launches;
    }
    void update(const OutOf &out, const Into &into, int route = -1) {
        if (rc) return;
        const pie_stack_norm &next = *into.norm, &post = out.norm;
        const int W = s->cfg.width, W64 = up64(W), WA = act_stride(W);
        const bool single = b.n_runs == b.n_rows;
        if (plan.big && pointwise(post) && pointwise(next) && !out.bias && !out.after && into.mix < 0) {
            hipLaunchKernelGGL(k_point_residual, dim3((unsigned)((W + 1023) / 1024), (unsigned)b.n_rows), dim3(256), 0, st, (const u16 *)s->y.p, W, norm_of(post), norm_of(next), s->x.p, W64,
                               (u16 *)s->h.p, WA, W);
            if (hipGetLastError() != hipSuccess) rc = pie::fail(PIE_E_HIP, "residual launch failed");
        } else {
            RowUpdateArgs a = {};
            a.y = plan.big ? (const void *)s->y.p : s->y32.p, a.y32 = !plan.big, a.ldy = plan.big ? W : W64, a.bias = out.bias, a.after = out.after, a.alpha = out.scale;
            if (into.mix >= 0 && single) a.mix = mix_args(into.mix);
            a.post = row_norm_of(post), a.next = row_norm_of(next), a.x = s->x.p, a.ldx = W64, a.h = s->h.p, a.ldh = WA, a.M = b.n_rows, a.W = W;
            if (route >= 0) a.route = s->route_dev.p + s->route_at[route], a.experts = s->layers[route].experts, a.router = (const u16 *)s->layers[route].w_router_rows, a.arrived = s->arrived.p;
            rc = row_update_launch(s->cfg.dtype, a, st);
        }
        ++launches;
        if (into.mix >= 0 && !single) token_mix(into.mix);
    }
    // a sublayer's last product [W, K], its norm, the residual sum and the next sublayer's norm
    void output(const void *w, const void *x, int ldx, int K, const OutOf &out, const Into &next, int route = -1) {
        const int W = s->cfg.width, W64 = up64(W), WA = act_stride(W), M = b.n_rows;
        if (plan.big) {
            gemm(w, x, ldx, M, W, K, s->y.p, W);
            return out.hyper ? streams(out.hyper, next) : update(out, next);
        }
        RowsArgs o = {};
        o.m = {(const char *)w, W, K, x, ldx, s->y32.p, W64};
        o.M = M;
        if (!out.hyper && pointwise(out.norm) && pointwise(*next.norm) && !out.bias && !out.after && route < 0 && next.mix < 0) {
            o.epi = ROWS_RESIDUAL, o.res = s->x.p, o.ld_res = W64, o.post = norm_of(out.norm), o.next = norm_of(*next.norm), o.h = s->h.p, o.ldh = WA;
            return linear(o);
        }
        o.epi = ROWS_SCALE_F32, o.scale = 1.0f;
        linear(o);
        if (out.hyper) streams(out.hyper, next);
        else update(out, next, route);
    }
    void linear(const RowsArgs &a, int batches = 1) {
        if (!rc) rc = rows_gemm_launch(s->cfg.dtype, a, batches, st), ++launches;
    }
};

// y = x . W^T in the stack's dtype (x nullptr: h)
void project(Pass &p, const void *w, int N, void *y, const void *x = nullptr) {
    pie_stack *s = p.s;
    const int W = s->cfg.width, WA = act_stride(W);
    if (!x) x = s->h.p;
    if (p.plan.big) return p.gemm(w, x, WA, p.b.n_rows, N, W, y, N);
    RowsArgs a = {};
    a.m = {(const char *)w, N, W, x, WA, y, N};
    a.M = p.b.n_rows, a.epi = ROWS_STORE;
    p.linear(a);
}

// where a pass's queries of a latent layer are: [M][ld], head h at h * D8; their rotated parts (rot_dim > 0) at q_rot, same row stride
struct LatentQueries {
    const void *q, *q_rot;
    int ld;
    HeadFinish finish;
};
// Attention and output of a latent layer whose latents are in their pages, or (riders, few rows) get there, and whose queries are rotated, along with the first launch
void latent_attend(Pass &p, int li, const pie_stack_layer &L, const LatentQueries &q, const RowsArgs &riders, const Into &next, int route) {
    pie_stack *s = p.s;
    const pie_stack_batch &b = p.b;
    const int D8 = up8(L.dim), V8 = up8(L.vdim), R8 = up8(L.rank), T8 = up8(L.rot_dim), H = L.heads, KO = H * V8, LO = act_stride(KO), dt = s->cfg.dtype;
    const void *slab = b.slabs[own_cache(L) ? li : L.kv_from];
    const bool spell = p.plan.long_rows && spelled_out(L);
    const ShortPart sp = short_part(s, b, p.plan, L);
    const int M = sp.M, runs = sp.runs;
    if (M > 0) {  // the latent form
        RowsArgs k = riders;
        k.m = {(const char *)L.w_uk, L.rank, L.dim, q.q, q.ld, s->ql.p, H * R8};
        k.M = M, k.epi = ROWS_STORE, k.w_batch = rows_weight_bytes(dt, L.rank, L.dim), k.x_batch = D8, k.y_batch = R8;
        p.linear(k, H);
        LatentAttnArgs t = {};
        t.q = s->ql.p, t.ldq = R8, t.q_rot = q.q_rot, t.ld_rot = q.ld, t.finish = q.finish;
        t.slab = slab, t.table = b.table, t.table_width = b.table_width, t.n_pages = (int)b.n_pages, t.n_seqs = b.n_seqs, t.pos = b.pos;
        t.runs = (const RowRun *)b.runs, t.n_runs = runs, t.single = runs == M, t.row_seq = b.row_seq;
        t.n_tiles = sp.tiles;
        t.H = H, t.R = T8 ? R8 + T8 : L.rank, t.ldr = R8 + T8, t.M = M, t.window = L.window, t.scale = L.scale, t.splits = plan_splits(b, L, t.n_tiles), t.ws = s->attn_ws.p, t.out = s->oc.p;
        const bool merge = t.splits > 1 && M <= MERGE_ROWS && R8 <= MERGE_LDR && dt == PIE_BF16 && R8 + T8 <= 1024;  // few rows: the next launch merges the key splits itself
        t.combine = !merge;
        if (!p.rc) p.rc = latent_attn_launch(dt, t, p.st), p.launches += t.splits > 1 && !merge ? 2 : 1;
        RowsArgs v = {};
        v.m = {(const char *)L.w_uv, L.vdim, L.rank, s->oc.p, H * R8, s->o.p, LO};
        v.M = M, v.epi = ROWS_STORE, v.w_batch = rows_weight_bytes(dt, L.vdim, L.rank), v.x_batch = R8, v.y_batch = V8;
        if (merge) v.merge = {s->attn_ws.p, t.splits, M, H, R8, q.finish};
        p.linear(v, H);
    }
    if (spell && !p.rc) {
        const RowRun *lr = (const RowRun *)b.runs + p.plan.short_runs;
        const int n_long = b.n_runs - p.plan.short_runs, n_ctx = (int)plan_context(b, p.plan, L.window), nkv = H * (D8 + V8), LC = act_stride(R8 + T8);
        p.rc = latent_gather_launch(lr, n_long, n_ctx, L.window, b.table, b.table_width, b.n_seqs, (int)b.n_pages, slab, R8 + T8, s->ctx.p, LC, p.st);
        p.gemm(L.w_kv, s->ctx.p, LC, n_ctx, nkv, L.rank, s->kv.p, nkv);
        WindowAttnArgs w = {};
        w.q = (const u16 *)q.q, w.kv = (const u16 *)s->kv.p, w.out = (u16 *)s->o.p, w.ld_q = q.ld, w.ld_kv = nkv, w.ld_out = LO, w.H = H, w.D8 = D8, w.V8 = V8, w.window = L.window;
        w.q_rot = (const u16 *)q.q_rot, w.k_rot = (const u16 *)s->ctx.p + R8, w.T8 = T8, w.ld_krot = LC, w.finish = q.finish, w.scale = L.scale, w.runs = lr, w.n_runs = n_long;
        int tiles = 0;
        for (int i = p.plan.short_runs; i < b.n_runs; ++i) tiles += (b.runs_host[4 * i + 1] + 127) / 128;
        if (!p.rc) p.rc = window_attn_launch(w, tiles, p.st), p.launches += 2;
    }
    p.output(L.w_o, s->o.p, LO, KO, out_of(L, L.post1, L.hyper1, nullptr), next, route);
}

// queries straight from the layer's input
void latent_mixer(Pass &p, int li, const pie_stack_layer &L, const Into &next, int route) {
    pie_stack *s = p.s;
    const pie_stack_batch &b = p.b;
    const int W = s->cfg.width, W64 = up64(W), WA = act_stride(W), D8 = up8(L.dim), R8 = up8(L.rank), H = L.heads, NI = H * D8 + R8;
    // many rows: q and the latents as two products where the tile rows allow it (together they are a little more than a round of workgroups)
    const bool two = p.plan.big && (H * D8) % 32 == 0;
    const int LQ = two ? H * D8 : NI;  // row stride of q
    if (two) {
        p.gemm(L.w_in, s->h.p, WA, b.n_rows, H * D8, W, s->q.p, LQ);
        p.gemm((const char *)L.w_in + (size_t)(H * D8 / 32) * (W64 / 64) * 4096, s->h.p, WA, b.n_rows, R8, W, s->c_raw.p, R8);
    } else if (p.plan.big) {
        p.gemm(L.w_in, s->h.p, WA, b.n_rows, NI, W, s->q.p, NI);
    } else {
        RowsArgs a = {};
        a.m = {(const char *)L.w_in, NI, W, s->h.p, WA, s->q.p, NI};
        a.M = b.n_rows, a.epi = ROWS_SPLIT, a.split = H * D8, a.y2 = s->c_raw.p, a.ldy2 = R8;
        p.linear(a);
    }
    if (p.rc) return;
    const LatentAppend append = {p.plan.big && !two ? (const void *)((const u16 *)s->q.p + H * D8) : s->c_raw.p, p.plan.big, p.plan.big && !two ? NI : R8, L.c_norm, L.eps, b.n_rows,
                                 L.rank, R8, b.pos, b.row_seq, b.table, b.table_width, (int)b.n_pages, b.n_seqs, b.slabs[li]};
    if (p.plan.big) p.rc = latent_append_launch(s->cfg.dtype, append, p.st), ++p.launches;  // (few rows: rides in the next launch)
    RowsArgs riders = {};
    if (!p.plan.big) riders.append = append;
    latent_attend(p, li, L, {s->q.p, nullptr, LQ, {}}, riders, next, route);
}

// queries out of a latent of their own, with rotated parts
void latent_query_mixer(Pass &p, int li, const pie_stack_layer &L, const Into &next, int route) {
    pie_stack *s = p.s;
    const pie_stack_batch &b = p.b;
    const int D8 = up8(L.dim), T8 = up8(L.rot_dim), H = L.heads, NI = in_columns(L), NQ = H * (D8 + T8), CQ = act_stride(L.q_rank), dt = s->cfg.dtype;
    project(p, L.w_in, NI, s->q.p);
    if (p.rc) return;
    LatentPrepArgs a = {};
    a.raw = s->q.p, a.ld = NI, a.M = b.n_rows, a.Q = L.q_rank, a.Q8 = up8(L.q_rank), a.R = L.rank, a.R8 = up8(L.rank), a.T = L.rot_dim, a.T8 = T8;
    a.q_norm = L.q_norm, a.c_norm = L.c_norm, a.eps = L.eps, a.rot = {L.rot_freq, L.rot_dims, L.rot_gain}, a.own = own_cache(L);
    a.pos = b.pos, a.row_seq = b.row_seq, a.table = b.table, a.table_width = b.table_width, a.n_pages = (int)b.n_pages, a.n_seqs = b.n_seqs;
    a.cq = s->cq.p, a.ldc = CQ, a.slab = b.slabs[li];
    char *q_rot = (char *)s->qu.p + (size_t)H * D8 * esize(s);
    const RotateArgs rotate = {q_rot, NQ, T8, H, b.n_rows, a.rot, b.pos};
    RowsArgs riders = {};
    const bool few = !p.plan.big && dt == PIE_BF16 && b.n_rows <= 16 && !L.q_norm;  // the norm rides in the queries' product, cache and rotation in the one behind it
    if (few) {
        if (a.own) riders.cache = a;
        if (L.rot_dims > 0) riders.rotate = rotate;
    } else p.rc = latent_prep_launch(dt, a, p.st), ++p.launches;
    if (p.plan.big) p.gemm(L.w_uq, s->cq.p, CQ, b.n_rows, NQ, L.q_rank, s->qu.p, NQ);
    else {
        RowsArgs u = {};
        u.m = {(const char *)L.w_uq, NQ, L.q_rank, few ? s->q.p : s->cq.p, few ? NI : CQ, s->qu.p, NQ};
        u.M = b.n_rows, u.epi = ROWS_STORE, u.x_norm = few, u.x_eps = L.eps;
        p.linear(u);
    }
    if (p.rc) return;
    if (!few && L.rot_dims > 0) p.rc = rotate_heads_launch(dt, rotate, p.st), ++p.launches;
    const HeadFinish finish = {L.head_sink, L.out_gate ? (const char *)s->q.p + (size_t)(NI - up8(H)) * esize(s) : nullptr, NI};
    latent_attend(p, li, L, {s->qu.p, q_rot, NQ, finish}, riders, next, route);
}

// the attention of a layer whose projections are in s->q; its heads' outputs go to the front of s->o
void attend(Pass &p, int li, const pie_stack_layer &L, int LO) {
    pie_stack *s = p.s;
    const pie_stack_batch &b = p.b;
    const int NI = in_columns(L), dt = s->cfg.dtype;
    const bool own = L.kv_from < 0;
    const KvGeometry geo = geometry(L);
    void *slab = b.slabs[own ? li : L.kv_from];
    const PageTable pages = {b.table, b.table_width, (int)b.n_pages, b.n_seqs};
    if (p.rc) return;
    KvPrepArgs k = {};
    k.raw = s->q.p, k.ld = NI, k.M = b.n_rows, k.bias = (const u16 *)L.in_bias, k.geo = geo, k.own = own, k.value_norm = L.value_norm != 0, k.row_norm = L.row_norm != 0;
    k.q_norm = L.q_norm, k.k_norm = L.k_norm, k.eps = L.eps, k.freq = L.rot_freq, k.rot_dims = L.rot_dims, k.rot_gain = L.rot_gain;
    k.pos = b.pos, k.row_seq = b.row_seq, k.pages = pages, k.slab = slab;
    p.rc = kv_prep_launch(dt, k, p.st), ++p.launches;
    PageAttnArgs a = {};
    a.q = s->q.p, a.ldq = NI, a.slab = slab, a.pages = pages, a.geo = geo, a.pos = b.pos, a.row_seq = b.row_seq, a.runs = (const RowRun *)b.runs;
    a.window = L.window, a.chunk = L.chunk, a.distance = L.distance, a.far = L.far, a.head_sink = L.head_sink, a.out_scale = L.out_scale;
    a.scale = L.scale, a.sink = L.sink, a.out = s->o.p, a.ld_out = LO, a.ws = s->attn_ws.p;
    if (L.out_gate) {
        const int at = NI - up8(L.heads);
        a.gate = (const char *)s->q.p + at * esize(s), a.ldg = NI, a.gate_bias = L.in_bias ? (const u16 *)L.in_bias + at : nullptr;
    }
    const ShortPart sp = short_part(s, b, p.plan, L);
    a.n_runs = sp.runs, a.n_tiles = sp.tiles, a.M = sp.M, a.single = sp.runs == sp.M, a.splits = plan_splits(b, L, sp.tiles);
    if (!p.rc && sp.M > 0) p.rc = page_attn_launch(dt, a, p.st), p.launches += page_attn_mfma(dt, geo) && a.splits > 1 ? 2 : 1;
    if (!p.rc && sp.M < b.n_rows) {
        a.runs += sp.runs, a.n_runs = b.n_runs - sp.runs, a.n_tiles = 0, a.M = b.n_rows, a.single = false, a.splits = 1;
        for (int i = sp.runs; i < b.n_runs; ++i) a.n_tiles += page_attn_long_tiles(b.runs_host[4 * i + 1], geo);
        p.rc = page_attn_long_launch(a, p.st), ++p.launches;
    }
}

void attention_mixer(Pass &p, int li, const pie_stack_layer &L, const Into &next, int route) {
    const int KO = out_columns(L), LO = act_stride(KO);
    project(p, L.w_in, in_columns(L), p.s->q.p);
    attend(p, li, L, LO);
    p.output(L.w_o, p.s->o.p, LO, KO, out_of(L, L.post1, L.hyper1, L.o_bias), next, route);
}

// time mixing, alone or beside an attention over the same rows; the mixes of the rows with their predecessors are in s->mixes
void time_mixer(Pass &p, int li, const pie_stack_layer &L, const Into &next, int route) {
    pie_stack *s = p.s;
    const pie_stack_batch &b = p.b;
    const pie_stack_time_mix &t = L.time_mix;
    const bool beside = L.mixer == PIE_MIXER_ATTENTION;
    const int W = s->cfg.width, WA = act_stride(W), M = b.n_rows, N = time_mix_columns(L), R8 = up8(t.rank), KO = out_columns(L), LO = act_stride(KO), dt = s->cfg.dtype;
    const size_t E = esize(s), part = (size_t)M * N * E, mix = (size_t)M * WA * E;
    char *at[TIME_MIXES];  // r, k, v, gate, low-rank input of the decay
    for (int i = 0; i < TIME_MIXES; ++i) at[i] = s->mixed.p + i * part;
    const void *w[TIME_MIXES] = {t.w_r, t.w_k, t.w_v, t.w_gate, t.w_low};
    if (p.plan.big) {
        if (beside) project(p, L.w_in, in_columns(L), s->q.p);
        for (int i = 0; i < TIME_MIXES; ++i) project(p, w[i], i < 4 ? N : R8, at[i], s->mixes.p + i * mix);
    } else {
        RowsArgs a = {};
        a.M = M, a.epi = ROWS_STORE;
        if (beside) a.mats[a.n_mats++] = {(const char *)L.w_in, in_columns(L), W, s->h.p, WA, s->q.p, in_columns(L)};
        for (int i = 0; i < TIME_MIXES; ++i) a.mats[a.n_mats++] = {(const char *)w[i], i < 4 ? N : R8, W, s->mixes.p + i * mix, WA, at[i], i < 4 ? N : R8};
        p.linear(a, a.n_mats);
    }
    if (beside) attend(p, li, L, LO);
    if (p.rc) return;
    TimeMixArgs m = {};
    m.r = at[0], m.k = at[1], m.v = at[2], m.gate = at[3], m.low = at[4], m.ld = N, m.ld_low = R8, m.M = M, m.H = t.heads, m.D = t.dim, m.D8 = up8(t.dim), m.rank = t.rank, m.R8 = R8;
    m.w_decay = (const u16 *)t.w_decay, m.decay_bias = t.decay_bias, m.bonus = t.bonus, m.o_norm = t.o_norm, m.eps = L.eps, m.out_scale = t.out_scale;
    m.pos = b.pos, m.row_seq = b.row_seq, m.slots = b.slots, m.n_seqs = b.n_seqs, m.n_slots = (int)b.n_slots, m.runs = (const RowRun *)b.runs;
    m.state = b.states[li], m.slot_floats = state_layout(s, li).total, m.ws = s->rec_ws.p, m.o = s->rec_o.p, m.out = s->o.p + (size_t)(KO - N) * E, m.ld_out = LO;
    const ChunkPart cp = chunk_part(s, b, L);
    m.n_runs = cp.runs;
    if (cp.runs) p.rc = time_mix_step_launch(dt, m, 0, cp.rows, p.st), p.launches += t.dim > 128 ? 2 : 1;
    if (!p.rc && cp.chunks) {
        m.runs += cp.runs, m.n_runs = b.n_runs - cp.runs;
        p.rc = time_mix_chunks_launch(dt, m, cp.chunks, cp.rows, M - cp.rows, p.st), p.launches += time_mix_chunk_launches(cp.chunks, t.heads, t.dim);
    }
    p.output(L.w_o, s->o.p, LO, KO, out_of(L, L.post1, L.hyper1, L.o_bias), next, route);
}

void gated_delta_mixer(Pass &p, int li, const pie_stack_layer &L, const Into &next, int route) {
    pie_stack *s = p.s;
    const pie_stack_batch &b = p.b;
    const int NI = in_columns(L), KO = out_columns(L), LO = act_stride(KO), dt = s->cfg.dtype;
    project(p, L.w_in, NI, s->q.p);
    if (p.rc) return;
    const StateLayout at = state_layout(s, li);
    GatedDeltaArgs d = {};
    d.raw = s->q.p, d.ld = NI, d.M = b.n_rows, d.H = L.heads, d.G = L.kv_heads, d.D = L.dim, d.D8 = up8(L.dim), d.V = L.vdim, d.V8 = up8(L.vdim), d.H8 = up8(L.heads);
    d.conv = L.mix_conv, d.taps = L.mix_taps, d.ldw = gated_channels(L), d.decay_rate = L.decay_rate, d.decay_bias = L.decay_bias, d.o_norm = L.o_norm;
    d.scale = L.scale, d.unit_eps = L.unit_eps, d.eps = L.eps, d.pos = b.pos, d.row_seq = b.row_seq, d.slots = b.slots, d.n_seqs = b.n_seqs, d.n_slots = (int)b.n_slots;
    d.runs = (const RowRun *)b.runs, d.n_runs = b.n_runs, d.state = b.states[li], d.slot_floats = at.total, d.ring = at.ring, d.ws = s->rec_ws.p, d.o = s->rec_o.p, d.out = s->o.p, d.ld_out = LO;
    if (b.n_runs < b.n_rows) {
        d.mixed = s->mixed.p;
        int tiles = 0;
        for (int i = 0; i < b.n_runs; ++i) tiles += conv_tiles(b.runs_host[4 * i + 1]);
        p.rc = gated_delta_conv_launch(dt, d, tiles, p.st), ++p.launches;
    }
    const ChunkPart cp = chunk_part(s, b, L);
    d.n_runs = cp.runs;
    if (!p.rc && cp.runs) p.rc = gated_delta_step_launch(dt, d, 0, cp.rows, p.st), p.launches += L.vdim > 256 ? 2 : 1;
    if (!p.rc && cp.chunks) {
        d.runs += cp.runs, d.n_runs = b.n_runs - cp.runs;
        p.rc = gated_delta_chunks_launch(dt, d, cp.chunks, cp.rows, b.n_rows - cp.rows, p.st), p.launches += gated_delta_chunk_launches(cp.chunks, L.heads, L.dim);
    }
    p.output(L.w_o, s->o.p, LO, KO, out_of(L, L.post1, L.hyper1, nullptr), next, route);
}

// x += side_norm(w_side_proj (gelu(w_side_gate x) * the token's vector for this layer)); h (= x on the way in) = next(x)
void side_input(Pass &p, int li, const pie_stack_layer &L, const Into &next) {
    pie_stack *s = p.s;
    const int M = p.b.n_rows, W = s->cfg.width, WA = act_stride(W), D = s->cfg.side_dim, DA = act_stride(D);
    const TokenVectors side = {(const u16 *)s->cfg.side_embed, (size_t)s->cfg.n_layers * D, (size_t)li * D, p.b.ids, s->cfg.vocab};
    int ld = DA;
    if (p.plan.big) {
        const int D8 = up8(D);
        ld = up64(D);
        if (D8 == ld) p.gemm(L.w_side_gate, s->h.p, WA, M, D8, W, s->side.p, ld);
        else if (!p.rc) {  // (rows longer than the product: its plan must not split K)
            p.rc = w16l_act_launch(L.w_side_gate, s->h.p, WA, M, D, W, s->side.p, ld, MFMA_ACT_NONE, 0.0f, 0.0f, nullptr, p.st), ++p.launches;
        }
        if (p.rc) return;
        hipLaunchKernelGGL(k_side_gate, dim3((unsigned)(((size_t)M * D + 255) / 256)), dim3(256), 0, p.st, (u16 *)s->side.p, ld, side, M, D);
        if (hipGetLastError() != hipSuccess) p.rc = pie::fail(PIE_E_HIP, "side input launch failed");
        ++p.launches;
    } else {
        RowsArgs a = {};
        a.m = {(const char *)L.w_side_gate, D, W, s->h.p, WA, s->side.p, ld};
        a.M = M, a.epi = ROWS_GELU_SIDE, a.side = side;
        p.linear(a);
    }
    p.output(L.w_side_proj, s->side.p, ld, D, {L.side_norm, nullptr, nullptr, false, 1.0f}, next);
}

void delta_mixer(Pass &p, int li, const pie_stack_layer &L, const Into &next, int route) {
    pie_stack *s = p.s;
    const pie_stack_batch &b = p.b;
    const int NI = in_columns(L), KO = out_columns(L), LO = act_stride(KO);
    project(p, L.w_in, NI, s->q.p);
    if (p.rc) return;
    DeltaArgs d = {};
    d.raw = s->q.p, d.ld = NI, d.M = b.n_rows, d.H = L.heads, d.D = L.dim, d.D8 = up8(L.dim), d.rank = L.rank, d.R8 = up8(L.rank), d.bias = (const u16 *)L.in_bias;
    d.w_decay = (const u16 *)L.w_decay, d.decay_bias = L.decay_bias, d.o_norm = L.o_norm, d.decay_scale = L.decay_scale, d.unit_eps = L.unit_eps, d.eps = L.eps;
    d.pos = b.pos, d.row_seq = b.row_seq, d.slots = b.slots, d.n_seqs = b.n_seqs, d.n_slots = (int)b.n_slots, d.runs = (const RowRun *)b.runs, d.n_runs = b.n_runs;
    d.state = b.states[li], d.slot_floats = state_layout(s, li).total, d.out = s->o.p, d.ld_out = LO;
    const ChunkPart dp = chunk_part(s, b, L);
    d.ws = s->rec_ws.p, d.o = s->rec_o.p, d.n_runs = dp.runs;
    if (dp.runs) p.rc = delta_step_launch(s->cfg.dtype, d, p.st), ++p.launches;
    if (!p.rc && dp.chunks) {
        d.runs += dp.runs, d.n_runs = b.n_runs - dp.runs;
        p.rc = delta_chunks_launch(s->cfg.dtype, d, dp.chunks, dp.rows, b.n_rows - dp.rows, p.st), p.launches += delta_launches(dp.chunks, L.heads, L.dim);
    }
    p.output(L.w_o, s->o.p, LO, KO, out_of(L, L.post1, L.hyper1, nullptr), next, route);
}

RecurrentArgs recurrent_args(const Pass &p, int li, int ld) {
    const pie_stack_batch &b = p.b;
    return {p.s->q.p, ld, b.n_rows, b.pos, b.row_seq, b.slots, b.n_seqs, (int)b.n_slots, (const RowRun *)b.runs, b.n_runs, b.states[li], state_layout(p.s, li).total, p.s->rec_ws.p};
}

void mlstm_mixer(Pass &p, int li, const pie_stack_layer &L, const Into &next, int route) {
    pie_stack *s = p.s;
    const pie_stack_batch &b = p.b;
    const int NI = in_columns(L), KO = out_columns(L), LO = act_stride(KO), D8 = up8(L.dim), V8 = up8(L.vdim), H = L.heads, dt = s->cfg.dtype;
    project(p, L.w_in, NI, s->q.p);
    if (p.rc) return;
    MlstmArgs m = {recurrent_args(p, li, NI), L.gate_bias, H, L.dim, D8, L.vdim, V8, up8(H), L.scale, L.gate_cap, L.unit_eps, s->rec_o.p, s->rec_den.p};
    const ChunkPart cp = chunk_part(s, b, L);
    m.r.n_runs = cp.runs;
    if (cp.runs) p.rc = mlstm_step_launch(dt, m, p.st), ++p.launches;
    if (!p.rc && cp.chunks) {
        m.r.runs += cp.runs, m.r.n_runs = b.n_runs - cp.runs;
        p.rc = mlstm_chunks_launch(m, cp.chunks, p.st), p.launches += 4;
    }
    const HeadOutArgs h = {s->rec_o.p, s->rec_den.p, (const char *)s->q.p + (size_t)H * (2 * D8 + V8) * esize(s), nullptr, NI, H, L.vdim, V8, L.o_norm, L.eps, s->o.p, LO, false, false, 1.0f};
    if (!p.rc) p.rc = head_out_launch(dt, h, 0, b.n_rows, p.st), ++p.launches;
    p.output(L.w_o, s->o.p, LO, KO, out_of(L, L.post1, L.hyper1, nullptr), next, route);
}

void mingru_mixer(Pass &p, int li, const pie_stack_layer &L, const Into &next, int route) {
    pie_stack *s = p.s;
    const pie_stack_batch &b = p.b;
    const int NI = in_columns(L), KO = out_columns(L), LO = act_stride(KO), dt = s->cfg.dtype;
    project(p, L.w_in, NI, s->q.p);
    if (p.rc) return;
    MingruArgs m = {recurrent_args(p, li, NI), (const u16 *)L.in_bias, L.dim, up8(L.dim), s->o.p, LO};
    const ChunkPart cp = chunk_part(s, b, L);
    m.r.n_runs = cp.runs;
    if (cp.runs) p.rc = mingru_step_launch(dt, m, p.st), ++p.launches;
    if (!p.rc && cp.chunks) {
        m.r.runs += cp.runs, m.r.n_runs = b.n_runs - cp.runs;
        p.rc = mingru_chunks_launch(dt, m, cp.chunks, p.st), p.launches += 3;
    }
    p.output(L.w_o, s->o.p, LO, KO, out_of(L, L.post1, L.hyper1, nullptr), next, route);
}

void feed_forward(Pass &p, int li, const pie_stack_layer &L, const Into &into, bool routed) {  // routed: the experts have been chosen already
    pie_stack *s = p.s;
    const int M = p.b.n_rows, W = s->cfg.width, W64 = up64(W), WA = act_stride(W), F = L.ff_size, FA = act_stride(F), dt = s->cfg.dtype;
    const pie_stack_norm &next = *into.norm;
    if (is_dense(L)) {
        const bool relu = L.ff == PIE_FF_RELU2, gated = L.ff == PIE_FF_GEGLU;
        if (p.plan.big) {
            const int act = gated ? MFMA_ACT_GELU : relu ? MFMA_ACT_RELU2 : MFMA_ACT_XIELU;
            if (!p.rc) p.rc = w16l_act_launch(L.w_up, s->h.p, WA, M, gated ? 2 * F : F, W, s->act.p, FA, act, L.act_alpha, L.act_beta, gated ? L.up_bias : nullptr, p.st), ++p.launches;
        } else {
            RowsArgs u = {};
            u.m = {(const char *)L.w_up, gated ? 2 * F : F, W, s->h.p, WA, s->act.p, FA};
            u.M = M, u.epi = gated ? ROWS_GELU_MUL : relu ? ROWS_RELU2 : ROWS_XIELU, u.bias = gated ? (const u16 *)L.up_bias : nullptr, u.act_alpha = L.act_alpha, u.act_limit = L.act_beta;
            p.linear(u);
        }
        return p.output(L.w_down, s->act.p, FA, F, out_of(L, L.post2, L.hyper2, L.down_bias), into);
    }
    const RouteLayer &r = s->route[li];
    const int S = L.shared_size, SA = act_stride(S);
    const size_t gu_stride = rows_weight_bytes(dt, 2 * F, W), dn_stride = rows_weight_bytes(dt, W, F);
    const bool clipped = L.act == PIE_ACT_CLIPPED;
    if (L.ff == PIE_FF_ROUTED_MOE && !routed) {  // logits, then the choice and its row lists
        RowsArgs z = {};
        z.m = {(const char *)L.w_router, L.experts, W, s->h.p, WA, s->logits_e.p, up8(L.experts)};
        z.M = M, z.epi = ROWS_SCALE_F32, z.scale = 1.0f;
        p.linear(z);
        if (p.rc) return;
        const RouteLayer *dev = s->route_dev.p + s->route_at[li];
        const bool few = !p.plan.big && M <= ROUTE_FEW_ROWS;
        if (!few) {
            hipLaunchKernelGGL(k_route_pick, dim3((unsigned)((M + 3) / 4)), dim3(256), 0, p.st, dev, M);
            ++p.launches;
        }
        hipLaunchKernelGGL(k_route, dim3(1), dim3(few && M == 1 ? 64 : 1024), (size_t)2 * L.experts * 4, p.st, dev, p.b.ids, M, s->cfg.vocab, few);
        if (hipGetLastError() != hipSuccess) p.rc = pie::fail(PIE_E_HIP, "routing launch failed");
        ++p.launches;
    }
    CombineArgs c = {};
    c.part = s->part.p, c.part_s = s->part_s.p, c.ldp = W64, c.ldp_s = p.plan.big && !(W & 3) ? W : W64, c.place = r.place, c.weight = r.weight, c.top = L.top, c.W = W, c.gate = S ? L.shared_gate : nullptr;
    c.pre = norm_of(L.pre2), c.post = norm_of(L.post2), c.next = norm_of(next), c.x = s->x.p, c.ldx = W64, c.h = s->h.p, c.ldh = WA;
    const bool elementwise = pointwise(L.post2) && pointwise(next);
    const dim3 cg((unsigned)M), cb((unsigned)std::min(1024, ((W + 3) / 4 + 63) / 64 * 64));
    if (p.plan.big) {
        const int tr = route_tile_rows(M, L.top, L.experts), tm = route_max_tiles(M, L.top, L.experts), rb = route_block(M, L.top, L.experts);
        if (!p.rc) p.rc = w16l_grouped_launch(L.w_gate_up, gu_stride, s->h.p, WA, (size_t)M, r.list, r.tiles, tm, rb, tr, 2 * F, W, s->act_e.p, FA, clipped ? MFMA_ACT_CLIPPED : MFMA_ACT_SWIGLU, L.act_alpha, L.act_limit,
                                               p.st);
        if (!p.rc) p.rc = w16l_grouped_launch(L.w_expert_down, dn_stride, s->act_e.p, FA, (size_t)M * L.top, nullptr, r.tiles, tm, rb, tr, W, F, s->part.p, W64, MFMA_ACT_NONE, 0.0f, 0.0f, p.st);
        p.launches += 2;
        if (S) {
            p.gemm(L.s_gate_up, s->h.p, WA, M, 2 * S, W, s->act_s.p, SA, true);
            p.gemm(L.s_down, s->act_s.p, SA, M, W, S, s->part_s.p, c.ldp_s);
        }
        if (p.rc) return;
        if (elementwise) hipLaunchKernelGGL((k_moe_combine<ElemBF16, ElemBF16>), cg, cb, 0, p.st, c);
    } else {
        const int groups = (int)std::min((long)L.experts, (long)M * L.top) + (S ? 1 : 0);
        RowsArgs u = {};
        u.m = {(const char *)L.w_gate_up, 2 * F, W, s->h.p, WA, s->act_e.p, FA};
        u.M = M, u.epi = clipped ? ROWS_CLIP_MUL : ROWS_SILU_MUL, u.act_alpha = L.act_alpha, u.act_limit = L.act_limit, u.w_batch = gu_stride, u.active = r.active, u.offset = r.offset, u.list = r.list, u.gather = true;
        if (S) u.shared = {(const char *)L.s_gate_up, 2 * S, W, s->h.p, WA, s->act_s.p, SA};
        p.linear(u, groups);
        RowsArgs d = {};
        d.m = {(const char *)L.w_expert_down, W, F, s->act_e.p, FA, s->part.p, W64};
        d.M = M, d.epi = ROWS_SCALE_F32, d.scale = 1.0f, d.w_batch = dn_stride, d.active = r.active, d.offset = r.offset, d.list = r.list;
        if (S) d.shared = {(const char *)L.s_down, W, S, s->act_s.p, SA, s->part_s.p, W64};
        p.linear(d, groups);
        if (p.rc) return;
        if (!elementwise) {
        } else if (dt == PIE_F32) hipLaunchKernelGGL((k_moe_combine<ElemF32, ElemF32>), cg, cb, 0, p.st, c);
        else hipLaunchKernelGGL((k_moe_combine<ElemBF16, ElemF32>), cg, cb, 0, p.st, c);
    }
    if (!elementwise) {
        RowUpdateArgs a = {};
        a.y = s->part.p, a.y32 = !p.plan.big, a.ldy = W64, a.place = r.place, a.weight = r.weight, a.top = L.top;
        a.post = row_norm_of(L.post2), a.next = row_norm_of(next), a.x = s->x.p, a.ldx = W64, a.h = s->h.p, a.ldh = WA, a.M = M, a.W = W;
        p.rc = row_update_launch(dt, a, p.st);
    } else if (hipGetLastError() != hipSuccess) p.rc = pie::fail(PIE_E_HIP, "expert combine launch failed");
    ++p.launches;
}

int stack_enqueue(pie_stack *s, const pie_stack_batch &b, const Plan &plan, hipStream_t st) {
    const int M = b.n_rows, W = s->cfg.width, W64 = up64(W), WA = act_stride(W), V = s->cfg.vocab, n = s->cfg.n_layers, dt = s->cfg.dtype;
    Pass p{s, b, plan, st};
    if (s->n_table) {
        hipLaunchKernelGGL(k_route, dim3((unsigned)s->n_table), dim3(1024), (size_t)s->route_lds, st, s->route_dev.p, b.ids, M, V, false);
        PIE_LAUNCH_CHECK();
        ++p.launches;
    }
    // what sublayer 1 of layer i (n: the final norm) takes in, and sublayer 2
    const int S = s->cfg.streams;
    auto mixer_in = [&](int i) -> Into {
        if (i >= n) return {&s->cfg.final_norm, nullptr, -1, -1};
        return {&s->layers[i].pre1, s->layers[i].hyper1, s->layers[i].conv_taps > 0 ? i : -1, has_time_mix(s->layers[i]) ? i : -1};
    };
    const pie_stack_norm plain = {nullptr, nullptr, 0.0f, PIE_NORM_NONE};
    const u16 *positions = (const u16 *)s->cfg.positions;
    const pie_stack_norm &first = *mixer_in(0).norm;
    const dim3 ge((unsigned)((W + 1023) / 1024), (unsigned)M);
    if (S) p.streams(nullptr, mixer_in(0));
    else if (dt == PIE_F32)
        hipLaunchKernelGGL(k_stack_embed<ElemF32>, ge, dim3(256), 0, st, b.ids, (const u16 *)s->cfg.embed, V, W, s->cfg.embed_scale, positions, s->cfg.max_positions, b.pos, !pointwise(first), norm_of(first), s->x.p, W64,
                           (float *)s->h.p, WA);
    else
        hipLaunchKernelGGL(k_stack_embed<ElemBF16>, ge, dim3(256), 0, st, b.ids, (const u16 *)s->cfg.embed, V, W, s->cfg.embed_scale, positions, s->cfg.max_positions, b.pos, !pointwise(first), norm_of(first), s->x.p, W64,
                           (u16 *)s->h.p, WA);
    PIE_LAUNCH_CHECK();
    p.launches += !S;
    if (!S && first.kind == PIE_NORM_RMS) {
        RowUpdateArgs a = {};
        a.next = row_norm_of(first), a.x = s->x.p, a.ldx = W64, a.h = s->h.p, a.ldh = WA, a.M = M, a.W = W;
        p.rc = row_update_launch(dt, a, st), ++p.launches;
    }
    if (n && has_time_mix(s->layers[0])) p.token_mix(0);
    for (int i = 0; i < n && !p.rc; ++i) {
        const pie_stack_layer &L = s->layers[i];
        const bool side = L.w_side_gate != nullptr;
        const Into last = mixer_in(i + 1), after = side ? Into{&plain, nullptr, -1, -1} : last, next = L.ff == PIE_FF_NONE ? after : Into{&L.pre2, L.hyper2, -1, -1};
        // some rows: the launch that makes the router's input also chooses the experts (for very few rows, spreading the router over the chip takes less time)
        const bool routed = L.ff == PIE_FF_ROUTED_MOE && !plan.big && L.w_router_rows && M >= ROUTE_MIN_ROWS && M <= ROUTE_FEW_ROWS && (long)L.experts * W <= ROUTE_FEW_WEIGHTS && W <= 8192;
        const int route = routed ? i : -1;
        switch (L.mixer) {
            case PIE_MIXER_LATENT: L.q_rank ? latent_query_mixer(p, i, L, next, route) : latent_mixer(p, i, L, next, route); break;
            case PIE_MIXER_ATTENTION: has_time_mix(L) ? time_mixer(p, i, L, next, route) : attention_mixer(p, i, L, next, route); break;
            case PIE_MIXER_TIME_MIX: time_mixer(p, i, L, next, route); break;
            case PIE_MIXER_GATED_DELTA: gated_delta_mixer(p, i, L, next, route); break;
            case PIE_MIXER_DELTA: delta_mixer(p, i, L, next, route); break;
            case PIE_MIXER_MLSTM: mlstm_mixer(p, i, L, next, route); break;
            default: mingru_mixer(p, i, L, next, route); break;
        }
        if (L.ff != PIE_FF_NONE && !p.rc) feed_forward(p, i, L, after, routed);
        if (side && !p.rc) side_input(p, i, L, last);
        if (b.tap && !p.rc && S) p.rc = stream_sum_launch(s->x.p, W64, S, b.tap + (size_t)i * M * W, M, W, st);
        else if (b.tap && !p.rc)
            PIE_HIP_TRY(hipMemcpy2DAsync(b.tap + (size_t)i * M * W, (size_t)W * 4, s->x.p, (size_t)W64 * 4, (size_t)W * 4, (size_t)M, hipMemcpyDeviceToDevice, st));
    }
    if (b.n_want > 0) {
        RowsArgs a = {};
        a.m = {(const char *)s->cfg.head, V, W, s->h.p, WA, b.logits, V};
        a.M = b.n_want, a.epi = s->cfg.logit_cap > 0.0f ? ROWS_SOFTCAP : ROWS_SCALE_F32, a.scale = s->cfg.logit_scale, a.act_limit = s->cfg.logit_cap, a.rows = b.want;
        p.linear(a);
        if (!p.rc && b.next) {
            hipLaunchKernelGGL(k_f32_stats, dim3(ST_TILES, (unsigned)b.n_want), dim3(256), 0, st, b.logits, V, s->stats.p);
            PIE_LAUNCH_CHECK();
            hipLaunchKernelGGL(k_f32_finish, dim3(b.logprobs ? 32 : 1, (unsigned)b.n_want), dim3(256), 0, st, b.logits, V, s->stats.p, b.logprobs, b.next, b.advance,
                               b.ids, b.pos, b.history, b.history_len);
            PIE_LAUNCH_CHECK();
            p.launches += 2;
        }
    }
    s->launches = p.launches;
    return p.rc;
}

bool norm_ok(const pie_stack_norm &n) {
    return n.kind == PIE_NORM_NONE || (n.kind == PIE_NORM_DYN_TANH && n.w && n.b) || (n.kind == PIE_NORM_RMS && n.w);
}
int mixer_ok(const pie_stack *s, int i, const pie_stack_layer &L) {
    PIE_REQUIRE((L.mixer == PIE_MIXER_TIME_MIX || (L.heads > 0 && L.dim > 0 && L.w_in)) && L.w_o && norm_ok(L.pre1) && norm_ok(L.post1), PIE_E_ARG, "pie_stack_set_layer: missing mixer weights or sizes");
    if (has_time_mix(L)) {
        const pie_stack_time_mix &t = L.time_mix;
        PIE_REQUIRE(L.mixer == PIE_MIXER_ATTENTION || L.mixer == PIE_MIXER_TIME_MIX, PIE_E_ARG, "pie_stack_set_layer: time mixing runs alone or beside an attention");
        PIE_REQUIRE(t.dim > 0 && t.dim <= TIME_MIX_MAX_DIM && t.rank > 0 && t.rank <= TIME_MIX_MAX_RANK, PIE_E_SHAPE, "pie_stack_set_layer: bad sizes (time mixing: dim at most 256, rank at most 1024)");
        PIE_REQUIRE(t.w_r && t.w_k && t.w_v && t.w_gate && t.w_low && t.w_decay && t.mu && t.decay_bias && t.bonus && t.o_norm, PIE_E_ARG, "pie_stack_set_layer: missing time mixing weights");
        PIE_REQUIRE(!s->cfg.streams && L.pre1.kind == PIE_NORM_NONE, PIE_E_ARG, "pie_stack_set_layer: time mixing reads the residual itself");
    }
    if (L.norm_after) PIE_REQUIRE(!s->cfg.streams && L.pre1.kind == PIE_NORM_NONE && L.pre2.kind == PIE_NORM_NONE && !is_moe(L), PIE_E_ARG, "pie_stack_set_layer: norms behind the sum go with plain sublayer inputs and dense feed-forwards");
    if (L.w_side_gate) PIE_REQUIRE(s->cfg.side_embed && s->cfg.side_dim > 0 && !s->cfg.streams && L.w_side_proj && norm_ok(L.side_norm), PIE_E_ARG, "pie_stack_set_layer: a side input needs its table, projection and norm");
    if (L.mixer == PIE_MIXER_LATENT) {
        PIE_REQUIRE(L.vdim > 0 && L.rank > 0 && L.q_rank >= 0 && L.rot_dim >= 0 && latent_row(L) <= 2048, PIE_E_SHAPE, "pie_stack_set_layer: bad mixer sizes (kv_rank + rot_dim at most 2048)");
        PIE_REQUIRE(L.w_uk && L.w_uv && (L.c_norm || !own_cache(L)), PIE_E_ARG, "pie_stack_set_layer: missing mixer weights");
        PIE_REQUIRE(L.q_rank ? L.w_uq != nullptr : !L.rot_dim && !L.out_gate && !L.head_sink, PIE_E_ARG,
                    "pie_stack_set_layer: rotation, gate and sink of latent attention go with a query latent, which needs its weights");
        PIE_REQUIRE(L.rot_dims >= 0 && L.rot_dims <= L.rot_dim && L.rot_dims % 2 == 0 && (L.rot_dims == 0 || L.rot_freq), PIE_E_SHAPE, "pie_stack_set_layer: bad rotation");
        if (!own_cache(L)) {
            PIE_REQUIRE(L.kv_from < i && s->have[L.kv_from], PIE_E_ARG, "pie_stack_set_layer: kv_from names an earlier layer");
            const pie_stack_layer &F = s->layers[L.kv_from];
            PIE_REQUIRE(F.mixer == PIE_MIXER_LATENT && own_cache(F) && F.rank == L.rank && F.rot_dim == L.rot_dim, PIE_E_SHAPE,
                        "pie_stack_set_layer: kv_from names a latent layer with a cache of its own, of the same sizes");
        }
    } else if (L.mixer == PIE_MIXER_TIME_MIX) {
        PIE_REQUIRE(has_time_mix(L), PIE_E_SHAPE, "pie_stack_set_layer: time mixing without heads");
    } else if (L.mixer == PIE_MIXER_GATED_DELTA) {
        PIE_REQUIRE(L.kv_heads > 0 && L.heads % L.kv_heads == 0 && L.dim <= GATED_MAX_DIM && L.vdim > 0 && L.vdim <= HEAD_OUT_MAX_DIM, PIE_E_SHAPE,
                    "pie_stack_set_layer: bad mixer sizes (gated delta rule: dim at most 256, vdim at most 2048, heads a multiple of kv_heads)");
        PIE_REQUIRE(L.mix_taps > 0 && L.mix_taps <= CONV_MAX_TAPS && L.mix_conv, PIE_E_SHAPE, "pie_stack_set_layer: a convolution of 1 .. 16 taps, with its weights");
        PIE_REQUIRE(L.decay_rate && L.decay_bias && L.o_norm, PIE_E_ARG, "pie_stack_set_layer: missing mixer weights");
    } else if (L.mixer == PIE_MIXER_ATTENTION) {
        PIE_REQUIRE(L.chunk >= 0 && (!L.chunk || L.window <= 0) && (!L.distance || L.far >= 0) && (!L.head_sink || L.sink == 0.0f), PIE_E_ARG, "pie_stack_set_layer: a window or chunks, and one kind of sink");
        PIE_REQUIRE(!L.row_norm || (L.dim == L.vdim && !L.rot_dims && !L.value_norm && L.q_norm && L.k_norm && L.kv_from < 0), PIE_E_SHAPE,
                    "pie_stack_set_layer: norms over all heads go with values that are the layer's own keys, without rotation");
        PIE_REQUIRE(L.vdim > 0 && L.kv_heads > 0 && L.heads % L.kv_heads == 0 && L.dim <= PAGE_ATTN_ROWS_DIM && L.vdim <= PAGE_ATTN_ROWS_DIM, PIE_E_SHAPE,
                    "pie_stack_set_layer: bad mixer sizes (heads of at most 1024 numbers, a multiple of kv_heads)");
        PIE_REQUIRE(L.rot_dims >= 0 && L.rot_dims <= L.dim && L.rot_dims % 2 == 0 && (L.rot_dims == 0 || L.rot_freq), PIE_E_SHAPE, "pie_stack_set_layer: bad rotation");
        if (L.kv_from >= 0) {
            PIE_REQUIRE(L.kv_from < i && s->have[L.kv_from], PIE_E_ARG, "pie_stack_set_layer: kv_from names an earlier layer");
            const pie_stack_layer &F = s->layers[L.kv_from];
            PIE_REQUIRE(F.mixer == PIE_MIXER_ATTENTION && F.kv_from < 0 && F.kv_heads == L.kv_heads && F.dim == L.dim && F.vdim == L.vdim, PIE_E_SHAPE,
                        "pie_stack_set_layer: kv_from names an attention layer with keys and values of its own, of the same sizes");
        }
    } else if (L.mixer == PIE_MIXER_DELTA) {
        PIE_REQUIRE(L.dim <= DELTA_MAX_DIM && L.rank > 0 && L.rank <= DELTA_MAX_RANK, PIE_E_SHAPE, "pie_stack_set_layer: bad mixer sizes (delta rule: dim at most 256, rank at most 1024)");
        PIE_REQUIRE(L.w_decay && L.decay_bias && L.o_norm, PIE_E_ARG, "pie_stack_set_layer: missing mixer weights");
        PIE_REQUIRE(L.decay_scale >= 0 && L.decay_scale <= DELTA_MAX_DECAY, PIE_E_ARG, "pie_stack_set_layer: decay_scale must be in [0, 2] (the chunk form divides by sixteen decays)");
    } else if (L.mixer == PIE_MIXER_MLSTM) {
        PIE_REQUIRE(L.vdim > 0 && L.dim <= MLSTM_MAX_DIM && L.vdim <= HEAD_OUT_MAX_DIM && L.gate_cap > 0, PIE_E_SHAPE, "pie_stack_set_layer: bad mixer sizes (mLSTM: dim at most 1024, vdim at most 2048)");
        PIE_REQUIRE(L.gate_bias && L.o_norm, PIE_E_ARG, "pie_stack_set_layer: missing mixer weights");
    } else if (L.mixer == PIE_MIXER_MINGRU) {
        PIE_REQUIRE(L.heads == 1, PIE_E_SHAPE, "pie_stack_set_layer: a minGRU has one head");
    } else PIE_REQUIRE(false, PIE_E_ARG, "pie_stack_set_layer: unknown mixer");
    if (s->cfg.streams) {
        PIE_REQUIRE(L.hyper1 && (L.ff == PIE_FF_NONE || L.hyper2) && L.post1.kind == PIE_NORM_NONE && (L.ff == PIE_FF_NONE || L.post2.kind == PIE_NORM_NONE) && !is_moe(L) && !L.o_bias, PIE_E_ARG,
                    "pie_stack_set_layer: hyper-connections need their weights, dense feed-forwards, and neither norms nor biases behind the sublayers");
        PIE_REQUIRE(L.conv_taps >= 0 && L.conv_taps <= CONV_MAX_TAPS && (!L.conv_taps || L.conv), PIE_E_SHAPE, "pie_stack_set_layer: a convolution of 1 .. 16 taps, with its weights");
    } else PIE_REQUIRE(!L.hyper1 && !L.hyper2 && !L.conv_taps, PIE_E_ARG, "pie_stack_set_layer: hyper-connections and convolutions go with several streams");
    return PIE_OK;
}

}  // namespace

extern "C" {

int pie_stack_create(const pie_stack_config *cfg, pie_stack **out) {
    PIE_REQUIRE(cfg && out, PIE_E_ARG, "pie_stack_create: null pointer");
    PIE_REQUIRE(cfg->dtype == PIE_BF16 || cfg->dtype == PIE_F32, PIE_E_ARG, "pie_stack_create: dtype must be PIE_BF16 or PIE_F32");
    PIE_REQUIRE(cfg->width > 0 && cfg->vocab > 0 && cfg->n_layers >= 0, PIE_E_SHAPE, "pie_stack_create: bad sizes");
    PIE_REQUIRE(cfg->embed && cfg->head && norm_ok(cfg->final_norm), PIE_E_ARG, "pie_stack_create: missing weights");
    PIE_REQUIRE(cfg->streams >= 0 && cfg->streams <= STREAMS_MAX && (cfg->streams == 0 || cfg->width <= ROW_UPDATE_MAX_WIDTH), PIE_E_SHAPE, "pie_stack_create: at most 16 streams, of at most 32768 numbers");
    PIE_REQUIRE((!cfg->positions || cfg->max_positions > 0) && (!cfg->bigram || (cfg->streams > 0 && cfg->buckets > 0 && cfg->n_layers > 0)), PIE_E_ARG,
                "pie_stack_create: position and bigram vectors need their sizes, and bigrams go with streams");
    PIE_REQUIRE(cfg->logit_cap >= 0.0f && (!cfg->side_embed || cfg->side_dim > 0), PIE_E_ARG, "pie_stack_create: bad logit cap or side vectors");
    pie_stack *s = new (std::nothrow) pie_stack();
    PIE_REQUIRE(s, PIE_E_HIP, "pie_stack_create: out of host memory");
    s->cfg = *cfg;
    s->layers.resize(cfg->n_layers), s->have.assign(cfg->n_layers, 0), s->route.assign(cfg->n_layers, RouteLayer{});
    *out = s;
    return PIE_OK;
}

int pie_stack_destroy(pie_stack *s) {
    delete s;
    return PIE_OK;
}

int pie_stack_set_layer(pie_stack *s, int i, const pie_stack_layer *L) {
    PIE_REQUIRE(s && L && i >= 0 && i < s->cfg.n_layers, PIE_E_ARG, "pie_stack_set_layer: bad argument");
    if (const int rc = mixer_ok(s, i, *L)) return rc;
    PIE_REQUIRE(L->ff == PIE_FF_NONE || (norm_ok(L->pre2) && norm_ok(L->post2) && L->ff_size > 0 && L->ff_size % 8 == 0 && L->shared_size % 8 == 0), PIE_E_ARG, "pie_stack_set_layer: missing feed-forward norms");
    if (is_dense(*L)) PIE_REQUIRE(L->w_up && L->w_down, PIE_E_ARG, "pie_stack_set_layer: missing dense weights");
    else if (is_moe(*L)) {
        PIE_REQUIRE(L->experts > 0 && L->experts <= 8192 && L->top > 0 && L->top <= L->experts, PIE_E_SHAPE, "pie_stack_set_layer: bad expert counts");
        PIE_REQUIRE((L->ff == PIE_FF_TABLE_MOE ? L->table != nullptr : L->w_router && L->correction) && L->w_gate_up && L->w_expert_down, PIE_E_ARG, "pie_stack_set_layer: missing expert weights");
        PIE_REQUIRE(L->act == PIE_ACT_SILU || L->act == PIE_ACT_CLIPPED, PIE_E_ARG, "pie_stack_set_layer: unknown activation");
        PIE_REQUIRE(L->shared_size == 0 || (L->shared_size > 0 && L->s_gate_up && L->s_down && L->shared_gate && L->act == PIE_ACT_SILU && pointwise(L->pre2) && pointwise(L->post2)),
                    PIE_E_ARG, "pie_stack_set_layer: a shared expert needs its weights, SiLU and element-wise norms");
    } else PIE_REQUIRE(L->ff == PIE_FF_NONE, PIE_E_ARG, "pie_stack_set_layer: unknown feed-forward");
    s->route[i] = RouteLayer{};
    if (is_moe(*L)) s->route[i].table = L->ff == PIE_FF_TABLE_MOE ? L->table : nullptr, s->route[i].correction = L->correction, s->route[i].top = L->top, s->route[i].experts = L->experts;
    s->route_rows = 0;
    s->layers[i] = *L, s->have[i] = 1;
    s->drop_graphs();
    return PIE_OK;
}

size_t pie_logprobs_argmax_f32_workspace(int rows) { return rows > 0 ? (size_t)rows * ST_TILES * sizeof(RowStat) : 0; }
int pie_logprobs_argmax_f32(const float *logits, int rows, int V, float *logprobs, int32_t *tokens, void *workspace, void *stream) {
    PIE_REQUIRE(logits && tokens && workspace, PIE_E_ARG, "pie_logprobs_argmax_f32: null pointer");
    PIE_REQUIRE(rows > 0 && rows <= 65535 && V > 0, PIE_E_SHAPE, "pie_logprobs_argmax_f32: bad shape");
    hipStream_t st = (hipStream_t)stream;
    hipLaunchKernelGGL(k_f32_stats, dim3(ST_TILES, (unsigned)rows), dim3(256), 0, st, logits, V, (RowStat *)workspace);
    hipLaunchKernelGGL(k_f32_finish, dim3(logprobs ? 32 : 1, (unsigned)rows), dim3(256), 0, st, logits, V, (const RowStat *)workspace, logprobs, tokens, 0, nullptr, nullptr, nullptr, 0);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

int pie_stack_page_row(const pie_stack *s, int i) {
    if (!s || i < 0 || i >= s->cfg.n_layers || !s->have[i]) return 0;
    const pie_stack_layer &L = s->layers[i];
    if (!own_cache(L)) return 0;
    return L.mixer == PIE_MIXER_LATENT ? latent_row(L) : (int)(geometry(L).page_elems() / PAGE_TOKENS);
}
size_t pie_stack_state_floats(const pie_stack *s, int i) {
    return s && i >= 0 && i < s->cfg.n_layers && s->have[i] ? state_layout(s, i).total : 0;
}
size_t pie_stack_page_bytes(const pie_stack *s, int i) { return (size_t)pie_stack_page_row(s, i) * PAGE_TOKENS * (s ? esize(s) : 0); }
int pie_stack_launches(const pie_stack *s) { return s ? s->launches : 0; }

int pie_stack_forward(pie_stack *s, const pie_stack_batch *bp, int flags, void *stream) {
    PIE_REQUIRE(s && bp, PIE_E_ARG, "pie_stack_forward: null pointer");
    const pie_stack_batch &b = *bp;
    hipStream_t st = (hipStream_t)stream;
    for (char h : s->have) PIE_REQUIRE(h, PIE_E_STATE, "pie_stack_forward: a layer has not been set");
    PIE_REQUIRE(b.n_rows > 0 && b.n_rows <= 65535 && b.n_seqs > 0 && b.table_width > 0 && b.n_runs > 0 && b.n_want >= 0 && b.n_pages > 0, PIE_E_SHAPE,
                "pie_stack_forward: a pass holds 1 .. 65535 rows of at least one sequence");
    PIE_REQUIRE(b.ids && b.pos && b.row_seq && b.table && b.runs && b.runs_host && b.slabs, PIE_E_ARG, "pie_stack_forward: null pointer");
    PIE_REQUIRE(b.n_want == 0 || b.logits, PIE_E_ARG, "pie_stack_forward: logits are asked for but have no buffer");
    PIE_REQUIRE(b.n_want <= b.n_rows && (b.want || b.n_want == 0 || b.n_want == b.n_rows), PIE_E_ARG, "pie_stack_forward: bad list of wanted rows");
    PIE_REQUIRE(!b.advance || (b.n_want == b.n_rows && !b.want && b.n_runs == b.n_rows && b.next), PIE_E_ARG, "pie_stack_forward: only a decode step can feed itself");
    int at = 0;
    for (int i = 0; i < b.n_runs; ++i) {
        const int32_t *r = b.runs_host + 4 * i;
        PIE_REQUIRE(r[0] == at && r[1] > 0 && r[2] >= 0 && r[2] < b.n_seqs, PIE_E_ARG, "pie_stack_forward: the runs must cover the rows in order");
        at += r[1];
    }
    PIE_REQUIRE(at == b.n_rows, PIE_E_ARG, "pie_stack_forward: the runs must cover the rows in order");
    for (int i = 0; i < s->cfg.n_layers; ++i) {
        PIE_REQUIRE(b.slabs[i] || !pie_stack_page_row(s, i), PIE_E_ARG, "pie_stack_forward: a layer has no pages");
        PIE_REQUIRE(!pie_stack_state_floats(s, i) || (b.slots && b.states && b.states[i] && b.n_slots > 0), PIE_E_ARG, "pie_stack_forward: a recurrent layer has no state slots");
    }
    const Plan plan = plan_pass(s, b);
    int rc = stack_reserve(s, b, plan, st);
    if (rc) return rc;
    size_t ws = 0;
    for (const pie_stack_layer &L : s->layers) ws = std::max(ws, attn_ws(s, b, plan, L));
    bool moved = false;
    if ((rc = s->attn_ws.need(ws, &moved))) return rc;
    if (moved) s->drop_graphs();
    if (!(flags & PIE_STEP_GRAPH) || b.tap) return stack_enqueue(s, b, plan, st);

    GraphKey key;
    key.b = b;
    key.b.slabs = nullptr, key.b.runs_host = nullptr, key.b.states = nullptr;
    if (b.states) key.states.assign(b.states, b.states + s->cfg.n_layers);
    key.slabs.assign(b.slabs, b.slabs + s->cfg.n_layers), key.runs.assign(b.runs_host, b.runs_host + 4 * b.n_runs);
    GraphSlot *slot = nullptr;
    for (GraphSlot &g : s->graphs)
        if (g.key.same(key)) slot = &g;
    if (!slot) {  // first pass of this shape: runs as launches (and loads every kernel)
        if (s->graphs.size() >= 4) {
            size_t old = 0;
            for (size_t i = 1; i < s->graphs.size(); ++i)
                if (s->graphs[i].used < s->graphs[old].used) old = i;
            if (s->graphs[old].exec) (void)hipGraphExecDestroy(s->graphs[old].exec);
            s->graphs.erase(s->graphs.begin() + old);
        }
        s->graphs.push_back({key, nullptr, ++s->tick});
        return stack_enqueue(s, b, plan, st);
    }
    slot->used = ++s->tick;
    if (!slot->exec) {
        hipGraph_t graph = nullptr;
        hipStream_t cs = nullptr;
        PIE_HIP_TRY(hipStreamCreateWithFlags(&cs, hipStreamNonBlocking));
        hipError_t e = hipStreamBeginCapture(cs, hipStreamCaptureModeThreadLocal);
        if (e == hipSuccess) {
            rc = stack_enqueue(s, b, plan, cs);
            e = hipStreamEndCapture(cs, &graph);
        }
        if (e == hipSuccess && !rc) e = hipGraphInstantiate(&slot->exec, graph, nullptr, nullptr, 0);
        if (graph) (void)hipGraphDestroy(graph);
        (void)hipStreamDestroy(cs);
        if (rc) return rc;
        PIE_HIP_TRY(e);
    }
    PIE_HIP_TRY(hipGraphLaunch(slot->exec, st));
    return PIE_OK;
}

}  // extern "C"
