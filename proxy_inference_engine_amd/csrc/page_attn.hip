// page_attn.hip -- softmax attention with grouped heads over paged keys and values (PIE_MIXER_ATTENTION): query / key norm, rotation, value norm, the page
// writes, and the attention itself with its denominator sink and per-head output gate.  What a query sees ends at a window or at the start of its chunk of positions; a score may
// have a learned number added that depends on the head and the key's distance.
//
// Keys and values lie in the pages in matrix-core operand order (KvGeometry), so an operand load is one contiguous KiB per wave, straight from memory to
// the registers that are the operand, or linearly through LDS: no swizzle, no transpose.
//   S^T[key, pair] = K . Q^T      A = keys (operand order), B = the pairs' queries, kept in registers      (v_mfma_f32_32x32x16_bf16)
//   online softmax in fp32, base 2; the reduction over keys runs over registers and one lane exchange
//   O^T[dim, pair] += V^T . P^T   A = values (operand order), B = the weights as the score layout leaves them, split into hi + lo bf16 halves (~16 bits)
// pair = (row of one run, head of one key/value head's group): what shares keys shares a tile.
//   short form: 32 pairs per workgroup; its four waves take turns at the 32-key blocks of the workgroup's key split and meet in LDS at the end;
//   long form:  128 pairs per workgroup, 32 per wave; pages staged through LDS by DMA, two buffers.
#include "mfma_store.hpp"    // w4m_pack
#include "prefill_attn.hpp"  // MfmaT, f32x16_t
#include "stack_types.hpp"

typedef __attribute__((ext_vector_type(4))) float pg_f32x4;

namespace {

constexpr float PG_NEG = -1e30f, PG_LOG2E = 1.44269504088896340736f;

// ---------------------------------------------------------------- projections -> queries, pages
// One wave per row and run of HB heads of one kind (queries, keys or values).  Lane l holds the dimension pairs l, l + 64, ... of a head; angles and places in a
// page are taken once for all heads of the wave.  NP: pairs per lane.
template <class E, int NP, int HB>
__global__ void __launch_bounds__(256) k_kv_prep(const KvPrepArgs a) {
    typedef typename E::type T;
    constexpr bool F32 = sizeof(T) == 4;
    const KvGeometry &geo = a.geo;
    const int nq = (geo.H + HB - 1) / HB, nk = a.own ? (geo.G + HB - 1) / HB : 0, lane = threadIdx.x & 63, m = blockIdx.x;
    int unit = __builtin_amdgcn_readfirstlane(blockIdx.y * 4 + (threadIdx.x >> 6));
    if (unit >= nq + 2 * nk) return;
    const bool is_q = unit < nq, is_v = unit >= nq + nk;
    unit -= is_q ? 0 : is_v ? nq + nk : nq;
    const int h0 = unit * HB, count = min(HB, (is_q ? geo.H : geo.G) - h0), n = is_v ? geo.vdim : geo.dim, stride = is_v ? geo.V8 : geo.D8;
    const int off = (is_q ? 0 : is_v ? (geo.H + geo.G) * geo.D8 : geo.H * geo.D8) + h0 * stride;
    T *x = (T *)a.raw + (size_t)m * a.ld + off;
    float u[HB][NP], v[HB][NP];
#pragma unroll
    for (int k = 0; k < HB; ++k)
#pragma unroll
        for (int j = 0; j < NP; ++j) {
            const int d = 2 * (lane + 64 * j), at = min(k, count - 1) * stride + min(d, (n - 1) & ~1);
            float p, r;  // (an odd head's last partner is its padding: zero)
            if constexpr (!F32) {
                const u32 w = *(const u32 *)(x + at);
                p = lo_f32<BF16>(w), r = hi_f32<BF16>(w);
            } else {
                const float2 w = *(const float2 *)(x + at);
                p = w.x, r = w.y;
            }
            if (a.bias) {
                const u32 w = *(const u32 *)(a.bias + off + at);  // (padded like the head)
                p += lo_f32<BF16>(w), r += hi_f32<BF16>(w);
            }
            u[k][j] = d < n ? p : 0.0f, v[k][j] = d + 1 < n ? r : 0.0f;
        }
    const int t = a.pos[m], tl = t & (PAGE_TOKENS - 1);
    T *page = is_q ? nullptr : (T *)a.slab + (size_t)page_of(a.pages, a.row_seq[m], t) * geo.page_elems() + h0 * geo.head_elems();
    const float *w = is_v ? nullptr : is_q ? a.q_norm : a.k_norm;
    const bool normed = is_v ? a.value_norm : w != nullptr;
    float sn[NP], cs[NP], wu[NP], wv[NP];
    int place[NP], place1[NP];
#pragma unroll
    for (int j = 0; j < NP; ++j) {
        const int d = 2 * (lane + 64 * j);
        sn[j] = 0.0f, cs[j] = 1.0f, wu[j] = wv[j] = 1.0f;
        if (w) wu[j] = w[min(d, n - 1)], wv[j] = w[min(d + 1, n - 1)];
        if (!is_v && d + 1 < a.rot_dims) {
            stack_sincos<F32>((float)t * a.freq[d >> 1], sn[j], cs[j]);
            sn[j] *= a.rot_gain, cs[j] *= a.rot_gain;
        }
        place[j] = is_q ? d : is_v ? geo.value(tl, d) : geo.key(tl, d), place1[j] = is_v ? geo.value(tl, d + 1) : 0;
    }
    const float inv_n = 1.0f / (float)n;
#pragma unroll
    for (int k = 0; k < HB; ++k) {
        if (k >= count) break;
        float inv = 1.0f;
        if (normed) {
            float ss = 0.0f;
#pragma unroll
            for (int j = 0; j < NP; ++j) ss = fmaf(u[k][j], u[k][j], fmaf(v[k][j], v[k][j], ss));
            ss = lanes_sum(ss) * inv_n + a.eps;
            inv = F32 ? 1.0f / sqrtf(ss) : __builtin_amdgcn_rsqf(ss);
        }
#pragma unroll
        for (int j = 0; j < NP; ++j) {
            const int d = 2 * (lane + 64 * j);
            if (d >= n) break;
            const float p = u[k][j] * inv * wu[j], r = v[k][j] * inv * wv[j];
            const float p2 = p * cs[j] - r * sn[j], r2 = r * cs[j] + p * sn[j];
            if (is_v) {
                T *dst = page + k * geo.head_elems();
                dst[place[j]] = E::pack(p);
                if (d + 1 < n) dst[place1[j]] = E::pack(r);
                continue;
            }
            T *dst = (is_q ? x + k * stride : page + k * geo.head_elems()) + place[j];  // (d even: both in one 8-dimension chunk, and the pair aligned)
            if constexpr (!F32) *(u32 *)dst = pack2<BF16>(p2, r2);
            else *(float2 *)dst = make_float2(p2, r2);
        }
    }
}

// One workgroup per row: the norms run over all heads of the row at once, and values are the keys in front of their norm.
template <class E>
__global__ void __launch_bounds__(256) k_kv_prep_row(const KvPrepArgs a) {
    typedef typename E::type T;
    __shared__ float s_red[2][4];
    const KvGeometry &geo = a.geo;
    const int m = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nq = geo.H * geo.D8, n = nq + (a.own ? geo.G * geo.D8 : 0);
    T *x = (T *)a.raw + (size_t)m * a.ld;
    struct Eight {
        float v[8];
    };
    auto eight = [&](int i) {  // with the bias (heads are padded to a multiple of 8 with zeros)
        Eight e;
        if constexpr (sizeof(T) == 2) {
            const uint4 w = *(const uint4 *)(x + i);
            const u32 u[4] = {w.x, w.y, w.z, w.w};
#pragma unroll
            for (int k = 0; k < 4; ++k) e.v[2 * k] = lo_f32<BF16>(u[k]), e.v[2 * k + 1] = hi_f32<BF16>(u[k]);
        } else {
#pragma unroll
            for (int k = 0; k < 8; ++k) e.v[k] = x[i + k];
        }
        if (a.bias) {
            const uint4 w = *(const uint4 *)(a.bias + i);
            const u32 u[4] = {w.x, w.y, w.z, w.w};
#pragma unroll
            for (int k = 0; k < 4; ++k) e.v[2 * k] += lo_f32<BF16>(u[k]), e.v[2 * k + 1] += hi_f32<BF16>(u[k]);
        }
        return e;
    };
    auto put = [&](T *p, const float (&v)[8]) {
        if constexpr (sizeof(T) == 2) *(uint4 *)p = make_uint4(pack2<BF16>(v[0], v[1]), pack2<BF16>(v[2], v[3]), pack2<BF16>(v[4], v[5]), pack2<BF16>(v[6], v[7]));
        else
#pragma unroll
            for (int k = 0; k < 8; ++k) p[k] = v[k];
    };
    constexpr int KEEP = 4;  // pieces of eight numbers per thread that stay in registers
    Eight kept[KEEP];
    float ss[2] = {0.0f, 0.0f};
#pragma unroll
    for (int j = 0; j < KEEP; ++j) {
        const int i = 8 * (threadIdx.x + 256 * j);
        if (i >= n) break;
        kept[j] = eight(i);
    }
    auto add = [&](int i, const Eight &e) {
        float s = 0.0f;
#pragma unroll
        for (int k = 0; k < 8; ++k) s = fmaf(e.v[k], e.v[k], s);
        if (i < nq) ss[0] += s;
        else ss[1] += s;
    };
    auto each = [&](auto &&f) {
#pragma unroll
        for (int j = 0; j < KEEP; ++j) {
            const int i = 8 * (threadIdx.x + 256 * j);
            if (i < n) f(i, kept[j]);
        }
        for (int i = 8 * (threadIdx.x + 256 * KEEP); i < n; i += 8 * 256) f(i, eight(i));
    };
    each(add);
    ss[0] = lanes_sum(ss[0]), ss[1] = lanes_sum(ss[1]);
    if (lane == 0) s_red[0][wave] = ss[0], s_red[1][wave] = ss[1];
    const int t = a.pos[m], tl = t & (PAGE_TOKENS - 1);
    T *page = (T *)a.slab + (size_t)page_of(a.pages, a.row_seq[m], t) * geo.page_elems();
    __syncthreads();
    float inv[2];
#pragma unroll
    for (int k = 0; k < 2; ++k) inv[k] = 1.0f / sqrtf(((s_red[k][0] + s_red[k][1]) + (s_red[k][2] + s_red[k][3])) / (float)((k ? geo.G : geo.H) * geo.dim) + a.eps);
    each([&](int i, const Eight &e) {
        const bool is_q = i < nq;
        const float *w = is_q ? a.q_norm + i : a.k_norm + i - nq;
        const float4 w0 = *(const float4 *)w, w1 = *(const float4 *)(w + 4);
        const float f = inv[!is_q];
        const float v[8] = {e.v[0] * f * w0.x, e.v[1] * f * w0.y, e.v[2] * f * w0.z, e.v[3] * f * w0.w, e.v[4] * f * w1.x, e.v[5] * f * w1.y, e.v[6] * f * w1.z, e.v[7] * f * w1.w};
        if (is_q) return put(x + i, v);
        const int g = (i - nq) / geo.D8, d = (i - nq) % geo.D8;
        T *head = page + g * geo.head_elems();
        put(head + geo.key(tl, d), v);
#pragma unroll
        for (int k = 0; k < 8; ++k)
            if (d + k < geo.vdim) head[geo.value(tl, d + k)] = E::pack(e.v[k]);
    });
}

// ---------------------------------------------------------------- common pieces
// the first position that a query at t sees
__device__ __forceinline__ int pg_first_key(const PageAttnArgs &a, int t) { return a.chunk > 0 ? t - t % a.chunk : a.window > 0 ? max(0, t - a.window + 1) : 0; }
struct PgTile {
    RowRun run;
    int g, gs, p0, live;  // key/value head, heads per group, first pair, live pairs
    __device__ __forceinline__ int row(int p) const { return run.row0 + (p0 + p) / gs; }
    __device__ __forceinline__ int head(int p) const { return g * gs + (p0 + p) % gs; }
};
template <int PAIRS>
__device__ __forceinline__ PgTile pg_tile(const PageAttnArgs &a, int index) {
    PgTile t;
    t.gs = a.geo.H / a.geo.G, t.g = index % a.geo.G;
    int i = index / a.geo.G, r = 0;
    if (a.single) {
        const int per_run = (t.gs + PAIRS - 1) / PAIRS;
        r = min(i / per_run, a.n_runs - 1), i %= per_run;
        t.run = RowRun{r, 1, a.row_seq[r], 0};
    } else {
        for (;;) {
            const int n = (a.runs[r].n_rows * t.gs + PAIRS - 1) / PAIRS;
            if (i < n || r + 1 >= a.n_runs) break;
            i -= n, ++r;
        }
        t.run = a.runs[r];
    }
    t.p0 = i * PAIRS;
    t.live = min(PAIRS, t.run.n_rows * t.gs - t.p0);
    return t;
}
__device__ __forceinline__ float pg_gate(const PageAttnArgs &a, bool is32, int row, int head) {
    if (!a.gate) return 1.0f;
    float z = is32 ? ((const float *)a.gate)[(size_t)row * a.ldg + head] : BF16::to_f32(((const u16 *)a.gate)[(size_t)row * a.ldg + head]);
    if (a.gate_bias) z += BF16::to_f32(a.gate_bias[head]);
    return 1.0f / (1.0f + expf(-z));
}

// What a head's sums are multiplied by at the end, when its weights are relative to the exponent m (base 2) and sum to l
__device__ __forceinline__ float pg_factor(const PageAttnArgs &a, bool is32, int row, int head, float m, float l) {
    const float gate = pg_gate(a, is32, row, head) * a.out_scale;
    if (a.head_sink) {
        const float s = a.head_sink[head] * PG_LOG2E, mm = fmaxf(m, s), f = __builtin_amdgcn_exp2f(m - mm);
        return gate * f / (l * f + __builtin_amdgcn_exp2f(s - mm));
    }
    return gate / (l + (a.sink > 0.0f ? a.sink * __builtin_amdgcn_exp2f(-m) : 0.0f));
}

// The numbers added to the scores by distance (PageAttnArgs::distance): the heads of one group, in LDS where they fit
constexpr int PG_TABLE = 3072;
enum { PG_PLAIN = 0, PG_NEAR_LDS = 1, PG_NEAR_GLOBAL = 2 };
struct PgDistance {
    const float *near;  // the pair's head: [far + 1]
    int far;
    float last;         // near[far], times log2 e
};
// group g's rows on their way into LDS: before anything else, a barrier in front of pg_distance()
template <int DIST>
__device__ __forceinline__ void pg_distance_load(const PageAttnArgs &a, int g, float *lds) {
    if constexpr (DIST == PG_NEAR_LDS) {
        const int n = a.geo.H / a.geo.G * (a.far + 1);
        const float *rows = a.distance + (size_t)g * n;
        for (int i = threadIdx.x; i < n; i += 256) lds[i] = rows[i];
    }
}
template <int DIST>
__device__ __forceinline__ PgDistance pg_distance(const PageAttnArgs &a, const PgTile &tile, int head, const float *lds) {
    if constexpr (DIST == PG_PLAIN) return {nullptr, 0, 0.0f};
    const int n = a.far + 1;
    if constexpr (DIST == PG_NEAR_LDS) __syncthreads();
    const float *near = DIST == PG_NEAR_LDS ? lds + (head - tile.g * tile.gs) * n : a.distance + (size_t)head * n;
    return {near, a.far, near[a.far] * PG_LOG2E};
}

// one 32-key block's scores -> weights: masks, moves the running maximum, splits the weights into bf16 halves
// near (DIST): keys of the block are nearer than the last row of the distance table
template <int DT, int DIST>
__device__ __forceinline__ void pg_softmax(const f32x16_t &s, bool masked, bool near, const PgDistance &dist, int t0, int h, int t_q, int t_min, float sl2, float &m_run, float &l_run,
                                           f32x16_t (&o)[DT], u32 (&hi)[8], u32 (&lo)[8]) {
    float sc[16], mloc = PG_NEG;
    if constexpr (DIST == PG_PLAIN) {
#pragma unroll
        for (int i = 0; i < 16; ++i) sc[i] = s[i] * sl2;
    } else if (near) {
#pragma unroll
        for (int i = 0; i < 16; ++i) sc[i] = fmaf(s[i], sl2, dist.near[min(max(t_q - (t0 + (i & 3) + 8 * (i >> 2) + 4 * h), 0), dist.far)] * PG_LOG2E);
    } else {
#pragma unroll
        for (int i = 0; i < 16; ++i) sc[i] = fmaf(s[i], sl2, dist.last);
    }
    if (masked) {
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const int t = t0 + (i & 3) + 8 * (i >> 2) + 4 * h;
            sc[i] = t <= t_q && t >= t_min ? sc[i] : PG_NEG;
        }
    }
#pragma unroll
    for (int i = 0; i < 16; ++i) mloc = fmaxf(mloc, sc[i]);
    mloc = xor32_max(mloc);
    // the running maximum moves only when a score exceeds it by 2^8: weights of up to 256 are as exact as weights of up to 1, and rescaling is rare
    if (__builtin_amdgcn_ballot_w64(mloc > m_run + 8.0f)) {
        const float mm = fmaxf(m_run, mloc), alpha = __builtin_amdgcn_exp2f(m_run - mm);
        l_run *= alpha;
#pragma unroll
        for (int d = 0; d < DT; ++d)
#pragma unroll
            for (int i = 0; i < 16; ++i) o[d][i] *= alpha;
        m_run = mm;
    }
#pragma unroll
    for (int i = 0; i < 16; i += 2) {
        const float pa = sc[i] > PG_NEG ? __builtin_amdgcn_exp2f(sc[i] - m_run) : 0.0f, pb = sc[i + 1] > PG_NEG ? __builtin_amdgcn_exp2f(sc[i + 1] - m_run) : 0.0f;
        l_run += pa + pb;
        const u32 w = w4m_pack<BF16>(pa, pb);
        hi[i >> 1] = w;
        lo[i >> 1] = w4m_pack<BF16>(pa - lo_f32<BF16>(w), pb - hi_f32<BF16>(w));
    }
}

// ---------------------------------------------------------------- short form
// KS, DT: upper bounds of D16 / 16 and V32 / 32 (FULL: heads are exactly that wide, and no load hangs on a branch)
template <int KS, int DT, int DIST, bool FULL>
__global__ void __launch_bounds__(256, DT <= 4 ? 2 : 1) k_page_attn(const PageAttnArgs a) {
    __shared__ __attribute__((aligned(16))) float s_o[4][DT * 4][64][4];
    __shared__ float s_m[4][32], s_l[4][32];
    const KvGeometry &geo = a.geo;
    const int D8 = FULL ? 16 * KS : geo.D8, D16 = FULL ? 16 * KS : geo.D16, V8 = FULL ? 32 * DT : geo.V8, V32 = FULL ? 32 * DT : geo.V32;
    pg_distance_load<DIST>(a, (int)blockIdx.x % geo.G, (float *)s_o);  // (the sums come there when nobody looks up distances any more)
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), c = lane & 31, h = lane >> 5;
    const PgTile tile = pg_tile<32>(a, blockIdx.x);
    if (tile.live <= 0) return;  // (a grid larger than the runs need)
    const int t_hi = a.pos[tile.row(tile.live - 1)], q_lo = a.pos[tile.row(0)], t_lo = pg_first_key(a, q_lo);
    const int first = t_lo / 32, nb = t_hi / 32 - first + 1, per = (nb + a.splits - 1) / a.splits;
    const int b_begin = first + (int)blockIdx.y * per, b_end = min(first + nb, b_begin + per);

    const int p = min(c, tile.live - 1), row = tile.row(p), head = tile.head(p);
    const int t_q = a.pos[row], t_min = pg_first_key(a, t_q);
    uint4 qf[KS];
#pragma unroll
    for (int s = 0; s < KS; ++s)
        qf[s] = FULL || 16 * s + 8 * h < D8 ? *(const uint4 *)((const u16 *)a.q + (size_t)row * a.ldq + head * D8 + 16 * s + 8 * h) : make_uint4(0, 0, 0, 0);

    const u16 *slab = (const u16 *)a.slab + tile.g * geo.head_elems() + lane * 8;
    const size_t page_elems = geo.page_elems();
    int pg_first = (b_begin + wave) / 2, pg = page_of(a.pages, tile.run.seq, (pg_first + lane) * PAGE_TOKENS);  // lane l: page pg_first + l of the sequence
    uint4 kf[KS], vf[DT][2];
    auto block = [&](int b) {
        const int bb = min(b, b_end - 1);
        int i = bb / 2 - pg_first;
        if (i >= 64) pg_first = bb / 2, i = 0, pg = page_of(a.pages, tile.run.seq, (pg_first + lane) * PAGE_TOKENS);
        return slab + (size_t)__builtin_amdgcn_readlane(pg, i) * page_elems;
    };
    auto load_k = [&](int b, const u16 *pp) {
#pragma unroll
        for (int s = 0; s < KS; ++s)
            if (FULL || 16 * s < D16) kf[s] = *(const uint4 *)(pp + (b & 1) * 32 * D16 + s * 512);
    };
    auto load_v = [&](int b, const u16 *pp) {
#pragma unroll
        for (int d = 0; d < DT; ++d)
            if (FULL || 32 * d < V32)
#pragma unroll
                for (int s = 0; s < 2; ++s) vf[d][s] = *(const uint4 *)(pp + PAGE_TOKENS * D16 + (b & 1) * 32 * V32 + d * 1024 + s * 512);
    };

    f32x16_t o[DT];
#pragma unroll
    for (int d = 0; d < DT; ++d)
#pragma unroll
        for (int i = 0; i < 16; ++i) o[d][i] = 0.0f;
    float m_run = PG_NEG, l_run = 0.0f;
    const float sl2 = a.scale * PG_LOG2E;
    if (b_begin + wave < b_end) {
        const u16 *pp = block(b_begin + wave);
        load_k(b_begin + wave, pp);
        load_v(b_begin + wave, pp);
    }
    const PgDistance dist = pg_distance<DIST>(a, tile, head, (const float *)s_o);
    for (int b = b_begin + wave; b < b_end; b += 4) {
        const int nx = min(b + 4, b_end - 1);
        const u16 *pn = block(nx);
        f32x16_t s0;
#pragma unroll
        for (int i = 0; i < 16; ++i) s0[i] = 0.0f;
#pragma unroll
        for (int s = 0; s < KS; ++s)
            if (FULL || 16 * s < D16) s0 = MfmaT<BF16>::run(kf[s], qf[s], s0);
        load_k(nx, pn);  // on its way during the softmax and the second product
        u32 hi[8], lo[8];
        pg_softmax<DT, DIST>(s0, true, q_lo - (b * 32 + 31) < dist.far, dist, b * 32, h, t_q, t_min, sl2, m_run, l_run, o, hi, lo);
#pragma unroll
        for (int d = 0; d < DT; ++d)
            if (FULL || 32 * d < V32)
#pragma unroll
                for (int s = 0; s < 2; ++s) {
                    o[d] = MfmaT<BF16>::run(vf[d][s], make_uint4(hi[4 * s], hi[4 * s + 1], hi[4 * s + 2], hi[4 * s + 3]), o[d]);
                    o[d] = MfmaT<BF16>::run(vf[d][s], make_uint4(lo[4 * s], lo[4 * s + 1], lo[4 * s + 2], lo[4 * s + 3]), o[d]);
                }
        load_v(nx, pn);
    }
    // the four waves' sums meet: each rescales its own to the common maximum, then every wave adds a quarter of the dimensions
    const float l_wave = xor32_sum(l_run);
    if (h == 0) s_m[wave][c] = m_run, s_l[wave][c] = l_wave;
    __syncthreads();
    float mx = PG_NEG, l = 0.0f;
#pragma unroll
    for (int w = 0; w < 4; ++w) mx = fmaxf(mx, s_l[w][c] > 0.0f ? s_m[w][c] : PG_NEG);
#pragma unroll
    for (int w = 0; w < 4; ++w) l += s_l[w][c] > 0.0f ? s_l[w][c] * __builtin_amdgcn_exp2f(s_m[w][c] - mx) : 0.0f;
    const float f = l_wave > 0.0f ? __builtin_amdgcn_exp2f(m_run - mx) : 0.0f;
#pragma unroll
    for (int d = 0; d < DT; ++d)
#pragma unroll
        for (int k = 0; k < 4; ++k)
            *(pg_f32x4 *)s_o[wave][4 * d + k][lane] = (pg_f32x4){o[d][4 * k] * f, o[d][4 * k + 1] * f, o[d][4 * k + 2] * f, o[d][4 * k + 3] * f};
    __syncthreads();
    if (c >= tile.live) return;
    const size_t pr = (size_t)row * geo.H + head, MH = (size_t)a.M * geo.H;
    float factor = 1.0f;
    if (a.splits == 1) factor = pg_factor(a, false, row, head, mx, l);
#pragma unroll
    for (int j = 0; j < DT; ++j) {
        const int q = wave * DT + j, d0 = 32 * (q >> 2) + 8 * (q & 3) + 4 * h;  // registers 4 k .. + 3 of block d <-> dims 32 d + 8 k + 4 h + {0 .. 3}
        if (d0 >= V8) continue;
        const pg_f32x4 v = (*(const pg_f32x4 *)s_o[0][q][lane] + *(const pg_f32x4 *)s_o[1][q][lane]) + (*(const pg_f32x4 *)s_o[2][q][lane] + *(const pg_f32x4 *)s_o[3][q][lane]);
        if (a.splits == 1)
            *(uint2 *)((u16 *)a.out + (size_t)row * a.ld_out + head * V8 + d0) = make_uint2(w4m_pack<BF16>(v[0] * factor, v[1] * factor), w4m_pack<BF16>(v[2] * factor, v[3] * factor));
        else
            *(pg_f32x4 *)(a.ws + ((size_t)blockIdx.y * MH + pr) * V32 + d0) = v;
    }
    if (a.splits > 1 && wave == 0 && h == 0) {
        float *ml = a.ws + (size_t)a.splits * MH * V32 + ((size_t)blockIdx.y * MH + pr) * 2;
        ml[0] = mx, ml[1] = l;
    }
}

// merges the key splits of one (row, head) pair
__global__ void __launch_bounds__(64) k_page_combine(const PageAttnArgs a) {
    const KvGeometry &geo = a.geo;
    const size_t pr = blockIdx.x, MH = (size_t)a.M * geo.H;
    const int row = (int)(pr / geo.H), head = (int)(pr % geo.H), lane = threadIdx.x;
    const float2 ml = lane < a.splits ? *(const float2 *)(a.ws + (size_t)a.splits * MH * geo.V32 + (lane * MH + pr) * 2) : make_float2(PG_NEG, 0.0f);
    const float mx = wave_max(ml.y > 0.0f ? ml.x : PG_NEG), f = ml.y > 0.0f ? __builtin_amdgcn_exp2f(ml.x - mx) : 0.0f;
    __shared__ float s_f[64];
    s_f[lane] = f * pg_factor(a, false, row, head, mx, wave_sum(ml.y * f));
    __syncthreads();
    const LatentMerge m = {a.ws, a.splits, a.M, geo.H, geo.V32};
    for (int d = lane * 4; d < geo.V8; d += 256) {
        const float4 v = latent_merge4(m, pr, d, [&](int s) { return s_f[s]; });
        *(uint2 *)((u16 *)a.out + (size_t)row * a.ld_out + head * geo.V8 + d) = make_uint2(pack2<BF16>(v.x, v.y), pack2<BF16>(v.z, v.w));
    }
}

// ---------------------------------------------------------------- long form
template <int KS, int DT, int DIST, bool FULL>
__global__ void __launch_bounds__(256, DT <= 4 ? 2 : 1) k_page_attn_long(const PageAttnArgs a) {
    constexpr int BUF = PAGE_TOKENS * (16 * KS + 32 * DT) * 2;
    __shared__ __attribute__((aligned(1024))) char s_kv[2 * BUF];
    __shared__ float s_near[DIST == PG_NEAR_LDS ? PG_TABLE : 1];
    const KvGeometry &geo = a.geo;
    const int D8 = FULL ? 16 * KS : geo.D8, D16 = FULL ? 16 * KS : geo.D16, V8 = FULL ? 32 * DT : geo.V8, V32 = FULL ? 32 * DT : geo.V32;
    pg_distance_load<DIST>(a, (int)blockIdx.x % geo.G, s_near);
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), c = lane & 31, h = lane >> 5;
    const PgTile tile = pg_tile<128>(a, (int)gridDim.x / geo.G * geo.G - geo.G - (int)blockIdx.x / geo.G * geo.G + (int)blockIdx.x % geo.G);  // later rows (more keys) first
    if (tile.live <= 0) return;
    const int t_last = tile.run.pos0 + (tile.p0 + tile.live - 1) / tile.gs, t_lo = pg_first_key(a, tile.run.pos0 + tile.p0 / tile.gs);
    const int g0 = t_lo / PAGE_TOKENS, g1 = t_last / PAGE_TOKENS;

    const int w0 = 32 * wave;
    const bool busy = w0 < tile.live;
    const int p = min(w0 + c, tile.live - 1), row = tile.row(p), head = tile.head(p);
    const int t_q = tile.run.pos0 + row - tile.run.row0, t_min = pg_first_key(a, t_q);
    const PgDistance dist = pg_distance<DIST>(a, tile, head, s_near);
    const int q_lo = tile.run.pos0 + (tile.p0 + min(w0, tile.live - 1)) / tile.gs, q_hi = tile.run.pos0 + (tile.p0 + min(w0 + 31, tile.live - 1)) / tile.gs;  // the wave's positions
    const int k_lo = pg_first_key(a, q_lo), k_full = pg_first_key(a, q_hi);
    uint4 qf[KS];
#pragma unroll
    for (int s = 0; s < KS; ++s)
        qf[s] = FULL || 16 * s + 8 * h < D8 ? *(const uint4 *)((const u16 *)a.q + (size_t)row * a.ldq + head * D8 + 16 * s + 8 * h) : make_uint4(0, 0, 0, 0);

    const unsigned lds0 = (unsigned)(size_t)(__attribute__((address_space(3))) void *)s_kv;
    const int units = (D16 + V32) / 8;  // KiB of a head's page
    int pg_first = g0, pg = page_of(a.pages, tile.run.seq, (pg_first + lane) * PAGE_TOKENS);
    auto fetch = [&](int g, int buf) {
        int i = g - pg_first;
        if (i >= 64) pg_first = g, i = 0, pg = page_of(a.pages, tile.run.seq, (pg_first + lane) * PAGE_TOKENS);
        const unsigned long long v = (unsigned long long)(uintptr_t)((const u16 *)a.slab + (size_t)__builtin_amdgcn_readlane(pg, i) * geo.page_elems() + tile.g * geo.head_elems());
        const unsigned long long src =
            (unsigned long long)(unsigned)__builtin_amdgcn_readfirstlane((int)(unsigned)v) | ((unsigned long long)(unsigned)__builtin_amdgcn_readfirstlane((int)(unsigned)(v >> 32)) << 32);
        for (int u = wave; u < units; u += 4) {
            const unsigned off = (unsigned)(u * 1024 + lane * 16), dst = lds0 + (unsigned)(buf * BUF + u * 1024);
            unsigned keep;
            asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %3\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, %2\n\ts_mov_b32 m0, %0"
                         : "=&s"(keep)
                         : "v"(off), "s"(src), "s"(dst)
                         : "memory");
        }
    };
    f32x16_t o[DT];
#pragma unroll
    for (int d = 0; d < DT; ++d)
#pragma unroll
        for (int i = 0; i < 16; ++i) o[d][i] = 0.0f;
    float m_run = PG_NEG, l_run = 0.0f;
    const float sl2 = a.scale * PG_LOG2E;
    fetch(g0, 0);
    for (int g = g0; g <= g1; ++g) {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();  // the page has landed for everyone, and nobody reads the other buffer any more
        if (g < g1) fetch(g + 1, (g - g0 + 1) & 1);
        const char *buf = s_kv + ((g - g0) & 1) * BUF;
#pragma unroll
        for (int half = 0; half < 2; ++half) {
            const int t0 = g * PAGE_TOKENS + 32 * half;
            if (!busy || t0 > q_hi || t0 + 31 < k_lo) continue;
            const char *kb = buf + half * 64 * D16 + lane * 16, *vb = buf + 2 * PAGE_TOKENS * D16 + half * 64 * V32 + lane * 16;
            f32x16_t s0;
#pragma unroll
            for (int i = 0; i < 16; ++i) s0[i] = 0.0f;
#pragma unroll
            for (int s = 0; s < KS; ++s)
                if (FULL || 16 * s < D16) s0 = MfmaT<BF16>::run(*(const uint4 *)(kb + s * 1024), qf[s], s0);
            u32 hi[8], lo[8];
            pg_softmax<DT, DIST>(s0, !(t0 + 31 <= q_lo && t0 >= k_full), q_lo - (t0 + 31) < dist.far, dist, t0, h, t_q, t_min, sl2, m_run, l_run, o, hi, lo);
#pragma unroll
            for (int d = 0; d < DT; ++d)
                if (FULL || 32 * d < V32)
#pragma unroll
                    for (int s = 0; s < 2; ++s) {
                        const uint4 v = *(const uint4 *)(vb + d * 2048 + s * 1024);
                        o[d] = MfmaT<BF16>::run(v, make_uint4(hi[4 * s], hi[4 * s + 1], hi[4 * s + 2], hi[4 * s + 3]), o[d]);
                        o[d] = MfmaT<BF16>::run(v, make_uint4(lo[4 * s], lo[4 * s + 1], lo[4 * s + 2], lo[4 * s + 3]), o[d]);
                    }
        }
    }
    const float l = xor32_sum(l_run);
    if (w0 + c >= tile.live) return;
    const float factor = pg_factor(a, false, row, head, m_run, l);
    u16 *dst = (u16 *)a.out + (size_t)row * a.ld_out + head * V8;
#pragma unroll
    for (int d = 0; d < DT; ++d)
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            const int d0 = 32 * d + 8 * k + 4 * h;
            if (d0 < V8)
                *(uint2 *)(dst + d0) = make_uint2(w4m_pack<BF16>(o[d][4 * k] * factor, o[d][4 * k + 1] * factor), w4m_pack<BF16>(o[d][4 * k + 2] * factor, o[d][4 * k + 3] * factor));
        }
}

// ---------------------------------------------------------------- one (row, head) per workgroup on the vector ALU: fp32 stacks and very wide heads
template <class E>
__global__ void __launch_bounds__(256) k_page_attn_rows(const PageAttnArgs a) {
    typedef typename E::type T;
    __shared__ float s_o[4][PAGE_ATTN_ROWS_DIM], s_q[PAGE_ATTN_ROWS_DIM], s_m[4], s_l[4];
    const KvGeometry &geo = a.geo;
    const int row = blockIdx.x, head = blockIdx.y, g = head / (geo.H / geo.G), lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    for (int d = threadIdx.x; d < geo.dim; d += 256) s_q[d] = E::load((const T *)a.q + (size_t)row * a.ldq + head * geo.D8 + d);
    for (int d = lane; d < geo.vdim; d += 64) s_o[wave][d] = 0.0f;
    __syncthreads();
    const int t_q = a.pos[row], t_lo = pg_first_key(a, t_q), seq = a.row_seq[row];
    const float *near = a.distance ? a.distance + (size_t)head * (a.far + 1) : nullptr;
    float m = PG_NEG, l = 0.0f;
    for (int t = t_lo + wave; t <= t_q; t += 4) {
        const T *kv = (const T *)a.slab + (size_t)page_of(a.pages, seq, t) * geo.page_elems() + g * geo.head_elems();
        const int tl = t & (PAGE_TOKENS - 1);
        float s = 0.0f;
        for (int d = lane; d < geo.dim; d += 64) s = fmaf(s_q[d], E::load(kv + geo.key(tl, d)), s);
        s = wave_sum(s) * a.scale;
        if (near) s += near[min(t_q - t, a.far)];
        const float m2 = fmaxf(m, s), f = expf(m - m2), w = expf(s - m2);
        l = l * f + w, m = m2;
        for (int d = lane; d < geo.vdim; d += 64) s_o[wave][d] = fmaf(w, E::load(kv + geo.value(tl, d)), s_o[wave][d] * f);
    }
    if (lane == 0) s_m[wave] = m, s_l[wave] = l;
    __syncthreads();
    float mx = fmaxf(fmaxf(s_m[0], s_m[1]), fmaxf(s_m[2], s_m[3]));
    if (a.head_sink) mx = fmaxf(mx, a.head_sink[head]);
    float f[4], sum = a.head_sink ? expf(a.head_sink[head] - mx) : a.sink > 0.0f ? a.sink * expf(-mx) : 0.0f;
#pragma unroll
    for (int w = 0; w < 4; ++w) f[w] = s_l[w] > 0.0f ? expf(s_m[w] - mx) : 0.0f, sum += s_l[w] * f[w];
    const float factor = pg_gate(a, sizeof(T) == 4, row, head) * a.out_scale / sum;
    for (int d = threadIdx.x; d < geo.vdim; d += 256)
        ((T *)a.out)[(size_t)row * a.ld_out + head * geo.V8 + d] = E::pack((s_o[0][d] * f[0] + s_o[1][d] * f[1] + s_o[2][d] * f[2] + s_o[3][d] * f[3]) * factor);
}

bool pg_lds_table(const PageAttnArgs &a) { return a.distance && (long)(a.geo.H / a.geo.G) * (a.far + 1) <= PG_TABLE; }
int pg_class(const KvGeometry &g) {  // 32-wide classes of the instantiations
    const int n = ((g.D16 + 31) / 32 * 32 > g.V32 ? (g.D16 + 31) / 32 : g.V32 / 32);
    return n <= 4 ? n : n <= 6 ? 6 : 8;
}

}  // namespace

int page_attn_tiles(int n_rows, const KvGeometry &g) { return (n_rows * (g.H / g.G) + 31) / 32 * g.G; }
int page_attn_long_tiles(int n_rows, const KvGeometry &g) { return (n_rows * (g.H / g.G) + 127) / 128 * g.G; }
size_t page_attn_ws_floats(int M, const KvGeometry &g, int splits) { return splits > 1 ? (size_t)splits * M * g.H * (g.V32 + 2) : 0; }
bool page_attn_mfma(int dtype, const KvGeometry &g) { return dtype == PIE_BF16 && g.dim <= PAGE_ATTN_MAX_DIM && g.vdim <= PAGE_ATTN_MAX_DIM; }

int kv_prep_launch(int dtype, const KvPrepArgs &a, hipStream_t st) {
    if (a.M <= 0) return PIE_OK;
    if (a.row_norm) {
        PIE_REQUIRE(a.q_norm && (a.k_norm || !a.own) && a.geo.dim == a.geo.vdim && a.rot_dims == 0 && !a.value_norm && a.ld % 8 == 0, PIE_E_SHAPE,
                    "paged attention: norms over all heads go with values that are the keys, without rotation");
        if (dtype == PIE_F32) hipLaunchKernelGGL(k_kv_prep_row<ElemF32>, dim3((unsigned)a.M), dim3(256), 0, st, a);
        else hipLaunchKernelGGL(k_kv_prep_row<ElemBF16>, dim3((unsigned)a.M), dim3(256), 0, st, a);
        PIE_LAUNCH_CHECK();
        return PIE_OK;
    }
    const int wide = a.geo.dim > a.geo.vdim ? a.geo.dim : a.geo.vdim;
    const int hb = a.M < 64 || wide > 256 ? 1 : wide > 128 ? 4 : 8;  // few rows: a wave per head
    auto units = [&](int n) { return (n + hb - 1) / hb; };
    const dim3 grid((unsigned)a.M, (unsigned)((units(a.geo.H) + (a.own ? 2 * units(a.geo.G) : 0) + 3) / 4));
#define PREP_GO(NP_, HB_) \
    if (dtype == PIE_F32) hipLaunchKernelGGL((k_kv_prep<ElemF32, NP_, HB_>), grid, dim3(256), 0, st, a); \
    else hipLaunchKernelGGL((k_kv_prep<ElemBF16, NP_, HB_>), grid, dim3(256), 0, st, a)
    if (wide <= 128) {
        if (hb == 1) { PREP_GO(1, 1); } else { PREP_GO(1, 8); }
    } else if (wide <= 256) {
        if (hb == 1) { PREP_GO(2, 1); } else { PREP_GO(2, 4); }
    } else { PREP_GO(8, 1); }
#undef PREP_GO
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

#define PG_CLASSES(GO) \
    switch (pg_class(a.geo)) { \
        case 1: { GO(2, 1); } break; \
        case 2: { GO(4, 2); } break; \
        case 3: { GO(6, 3); } break; \
        case 4: { GO(8, 4); } break; \
        case 6: { GO(12, 6); } break; \
        default: { GO(16, 8); } break; \
    }

int page_attn_launch(int dtype, const PageAttnArgs &a, hipStream_t st) {
    if (a.M <= 0) return PIE_OK;
    PIE_REQUIRE(a.geo.G > 0 && a.geo.H % a.geo.G == 0 && a.geo.dim > 0 && a.geo.vdim > 0 && a.geo.dim <= PAGE_ATTN_ROWS_DIM && a.geo.vdim <= PAGE_ATTN_ROWS_DIM, PIE_E_SHAPE,
                "paged attention: heads of at most 1024 numbers, a whole number of them per key/value head");
    if (!page_attn_mfma(dtype, a.geo)) {
        const dim3 grid((unsigned)a.M, (unsigned)a.geo.H);
        if (dtype == PIE_F32) hipLaunchKernelGGL(k_page_attn_rows<ElemF32>, grid, dim3(256), 0, st, a);
        else hipLaunchKernelGGL(k_page_attn_rows<ElemBF16>, grid, dim3(256), 0, st, a);
        PIE_LAUNCH_CHECK();
        return PIE_OK;
    }
    if (a.n_tiles <= 0) return PIE_OK;
    PIE_REQUIRE(a.splits >= 1 && a.splits <= 64 && (a.splits == 1 || a.ws), PIE_E_ARG, "paged attention: 1 .. 64 key splits, which need their workspace");
    PIE_REQUIRE(a.ldq % 8 == 0 && a.ld_out % 4 == 0, PIE_E_ALIGN, "paged attention: row strides");
    const dim3 grid((unsigned)a.n_tiles, (unsigned)a.splits);
    const bool lds_table = pg_lds_table(a);
#define PG_DIST(K_, D_, F_) \
    if (!a.distance) hipLaunchKernelGGL((k_page_attn<K_, D_, PG_PLAIN, F_>), grid, dim3(256), 0, st, a); \
    else if (lds_table) hipLaunchKernelGGL((k_page_attn<K_, D_, PG_NEAR_LDS, F_>), grid, dim3(256), 0, st, a); \
    else hipLaunchKernelGGL((k_page_attn<K_, D_, PG_NEAR_GLOBAL, false>), grid, dim3(256), 0, st, a)
#define PG_GO(K_, D_) \
    if (a.geo.D8 == 16 * K_ && a.geo.V8 == 32 * D_) { PG_DIST(K_, D_, true); } \
    else { PG_DIST(K_, D_, false); }
    PG_CLASSES(PG_GO)
#undef PG_GO
#undef PG_DIST
    PIE_LAUNCH_CHECK();
    if (a.splits > 1) {
        hipLaunchKernelGGL(k_page_combine, dim3((unsigned)(a.M * a.geo.H)), dim3(64), 0, st, a);
        PIE_LAUNCH_CHECK();
    }
    return PIE_OK;
}

int page_attn_long_launch(const PageAttnArgs &a, hipStream_t st) {
    if (a.n_tiles <= 0) return PIE_OK;
    PIE_REQUIRE(page_attn_mfma(PIE_BF16, a.geo) && a.ldq % 8 == 0 && a.ld_out % 4 == 0, PIE_E_SHAPE, "paged attention: the long form takes heads of up to 256 numbers");
    const dim3 grid((unsigned)a.n_tiles);
    const bool lds_table = pg_lds_table(a);
#define PG_DIST(K_, D_, F_) \
    if (!a.distance) hipLaunchKernelGGL((k_page_attn_long<K_, D_, PG_PLAIN, F_>), grid, dim3(256), 0, st, a); \
    else if (lds_table) hipLaunchKernelGGL((k_page_attn_long<K_, D_, PG_NEAR_LDS, F_>), grid, dim3(256), 0, st, a); \
    else hipLaunchKernelGGL((k_page_attn_long<K_, D_, PG_NEAR_GLOBAL, false>), grid, dim3(256), 0, st, a)
#define PG_GO(K_, D_) \
    if (a.geo.D8 == 16 * K_ && a.geo.V8 == 32 * D_) { PG_DIST(K_, D_, true); } \
    else { PG_DIST(K_, D_, false); }
    PG_CLASSES(PG_GO)
#undef PG_GO
#undef PG_DIST
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}
