// stack_types.hpp -- what the kernels of the layer-stack models share: the element types, the norms that ride in epilogues, and the operand
// descriptions of the row-wise Linear (rows_gemm.hip), the attentions (latent_attn.hip, window_attn.hip, page_attn.hip), the recurrences (delta_rule.hip, gated_delta.hip,
// time_mix.hip, mlstm.hip, mingru.hip) and what stands between sublayers (row_update.hip, stream_update.hip).
//
// Every activation row has a stride that is a multiple of 8 elements (act_stride(), or packed); a Linear reads 64 ceil(K / 64) elements of it.  The columns past K meet zero
// weights, so they only have to be finite: the owner zero-fills its buffers once and keeps 64 elements of slack behind each.
#pragma once
#include "common.hpp"

constexpr int PAGE_TOKENS = 64;
// Row stride (elements) of a 16-bit activation of K columns: an odd number of 256-byte lines, so that the same columns of consecutive rows -- what an
// MFMA operand load touches -- lie in different cache channels; at a stride of a power of two they would queue up in one.
static inline int act_stride(int K) { return ((K + 127) / 128 | 1) * 128; }

// Element types of a stack: 16-bit storage (MFMA products, fp32 accumulation) or fp32 throughout.
struct ElemBF16 {
    typedef u16 type;
    static __device__ __forceinline__ float load(const u16 *p) { return BF16::to_f32(*p); }
    static __device__ __forceinline__ u16 pack(float v) { return BF16::from_f32(v); }
};
struct ElemF32 {
    typedef float type;
    static __device__ __forceinline__ float load(const float *p) { return *p; }
    static __device__ __forceinline__ float pack(float v) { return v; }
};

// two neighbouring numbers
struct ElemPair {
    float x, y;
};
template <class E>
__device__ __forceinline__ ElemPair load_pair(const typename E::type *p) {
    if constexpr (sizeof(typename E::type) == 4) return {((const float2 *)p)->x, ((const float2 *)p)->y};
    else {
        const u32 w = *(const u32 *)p;
        return {lo_f32<BF16>(w), hi_f32<BF16>(w)};
    }
}

// A norm without statistics, applied element by element in fp32: w * tanh(alpha x) + b (Dynamic Tanh).  Because it needs no reduction over the row,
// the kernel that produces an element can apply both the norm behind its own sublayer and the norm in front of the next one.
struct PointNorm {
    const float *w, *b;
    float alpha;
};
// tanh to a few units in the last place: below 1/4 the odd Taylor polynomial (next term < 1e-8 of the value), above it 1 - 2 / (e^{2 |z|} + 1)
__device__ __forceinline__ float fast_tanh(float z) {
    const float a = fabsf(z), z2 = z * z;
    const float p = z * fmaf(z2, fmaf(z2, fmaf(z2, fmaf(z2, 62.0f / 2835.0f, -17.0f / 315.0f), 2.0f / 15.0f), -1.0f / 3.0f), 1.0f);
    const float e = __builtin_amdgcn_exp2f(a * 2.88539008177792681472f);  // e^{2 |z|}; infinite for large |z|: the quotient is then 0
    const float q = copysignf(1.0f - 2.0f * __builtin_amdgcn_rcpf(e + 1.0f), z);
    return a < 0.25f ? p : q;
}
__device__ __forceinline__ float point_norm(const PointNorm &n, int i, float x) { return fmaf(fast_tanh(n.alpha * x), n.w[i], n.b[i]); }

// four columns i .. i + 3 (i a multiple of 4; w and b hold a multiple of 4 elements)
__device__ __forceinline__ float4 point_norm4(const PointNorm &n, int i, float4 x) {
    const float4 w = *(const float4 *)(n.w + i), b = *(const float4 *)(n.b + i);
    return make_float4(fmaf(fast_tanh(n.alpha * x.x), w.x, b.x), fmaf(fast_tanh(n.alpha * x.y), w.y, b.y), fmaf(fast_tanh(n.alpha * x.z), w.z, b.z),
                       fmaf(fast_tanh(n.alpha * x.w), w.w, b.w));
}

// exp(x) and 1 / (1 + exp(-x)): fp32 stacks take the library's, 16-bit ones the exponential unit (a few units in the last place)
constexpr float STACK_LOG2E = 1.44269504088896340736f;
template <bool F32>
__device__ __forceinline__ float stack_exp(float x) {
    return F32 ? expf(x) : __builtin_amdgcn_exp2f(x * STACK_LOG2E);
}
template <bool F32>
__device__ __forceinline__ float stack_sigmoid(float x) {
    return F32 ? 1.0f / (1.0f + expf(-x)) : __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(x * -STACK_LOG2E));
}

template <bool F32>
__device__ __forceinline__ float stack_silu(float x) { return x * stack_sigmoid<F32>(x); }
template <bool F32>
__device__ __forceinline__ float stack_tanh(float x) { return F32 ? tanhf(x) : fast_tanh(x); }
// z / 2 (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3)))
template <bool F32>
__device__ __forceinline__ float gelu_tanh(float z) {
    constexpr float c = 0.79788456080286535588f;
    return 0.5f * z * (1.0f + stack_tanh<F32>(c * z * fmaf(0.044715f * z, z, 1.0f)));
}
// log(1 + e^z)
template <bool F32>
__device__ __forceinline__ float stack_softplus(float z) { return fmaxf(z, 0.0f) + log1pf(F32 ? expf(-fabsf(z)) : __builtin_amdgcn_exp2f(-fabsf(z) * STACK_LOG2E)); }

// sin and cos of an angle: the library's in fp32 stacks; else reduced to one turn in two steps, then the trigonometric unit (absolute error about 1e-6)
template <bool F32>
__device__ __forceinline__ void stack_sincos(float a, float &s, float &c) {
    if constexpr (F32) sincosf(a, &s, &c);
    else {
        const float n = rintf(a * 0.15915494309189533577f), r = fmaf(n, 1.7484556e-7f, fmaf(n, -6.2831855f, a)) * 0.15915494309189533577f;  // (6.2831855f is 2 pi + 1.7484556e-7)
        s = __builtin_amdgcn_sinf(r), c = __builtin_amdgcn_cosf(r);
    }
}

// up z^2 + z / 2 for z > 0, down (e^z - 1 - z) + z / 2 for z <= 0 (xIELU); e^z - 1 - z by its series near zero, where the difference would cancel
template <bool F32>
__device__ __forceinline__ float xielu(float z, float up, float down) {
    const float n = fminf(z, 0.0f);
    if constexpr (!F32) {  // (the difference's absolute error of 1e-7 is below what the result is rounded to)
        const float p = fmaxf(z, 0.0f), e = __builtin_amdgcn_exp2f(n * STACK_LOG2E);
        return fmaf(p, fmaf(up, p, 0.5f), fmaf(0.5f - down, n, fmaf(down, e, -down)));
    }
    const float series = 0.5f * n * n * fmaf(n * (1.0f / 3.0f), fmaf(n * 0.25f, fmaf(n * 0.2f, fmaf(n * (1.0f / 6.0f), fmaf(n * (1.0f / 7.0f), 1.0f, 1.0f), 1.0f), 1.0f), 1.0f), 1.0f);
    const float g = n > -0.25f ? series : stack_exp<F32>(n) - 1.0f - n;
    return fmaf(0.5f, z, z > 0.0f ? up * z * z : down * g);
}

// sum / maximum over the wave without LDS, in every lane
__device__ __forceinline__ float lanes_sum(float v) { return xor32_sum(xor16_sum(lanes16_sum(v))); }
__device__ __forceinline__ float lanes_max(float v) {
    v = fmaxf(v, __builtin_amdgcn_update_dpp(v, v, 0xB1, 0xF, 0xF, true));   // quad_perm [1,0,3,2]
    v = fmaxf(v, __builtin_amdgcn_update_dpp(v, v, 0x4E, 0xF, 0xF, true));   // quad_perm [2,3,0,1]
    v = fmaxf(v, __builtin_amdgcn_update_dpp(v, v, 0x141, 0xF, 0xF, true));  // row_half_mirror
    v = fmaxf(v, __builtin_amdgcn_update_dpp(v, v, 0x140, 0xF, 0xF, true));  // row_mirror
    return xor32_max(xor16_max(v));
}

// ---------------------------------------------------------------- latent append
// c_raw [M][ldc], fp32 or (raw16) bf16 -> RMS norm with weight w -> the row of its page
struct LatentAppend {
    const void *c_raw;
    bool raw16;
    int ldc;
    const float *w;
    float eps;
    int M, R, ldr;
    const int *pos, *row_seq, *table;
    int table_width, n_pages, n_seqs;
    void *slab;
};
template <class E, class X, int THREADS>
__device__ __forceinline__ void latent_append_row(const LatentAppend &a, int m, float *red) {  // red: THREADS / 64 floats of LDS
    const typename X::type *x = (const typename X::type *)a.c_raw + (size_t)m * a.ldc;
    const int t = a.pos[m], j = min(t / PAGE_TOKENS, a.table_width - 1);
    float ss = 0.0f;
    for (int r = threadIdx.x; r < a.R; r += THREADS) {
        const float v = X::load(x + r);
        ss = fmaf(v, v, ss);
    }
    ss = wave_sum(ss);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    const size_t page = min((unsigned)a.table[(size_t)min(a.row_seq[m], a.n_seqs - 1) * a.table_width + j], (unsigned)a.n_pages - 1u);
    __syncthreads();
    float sum = red[0];
#pragma unroll
    for (int i = 1; i < THREADS / 64; ++i) sum += red[i];
    const float inv = 1.0f / sqrtf(sum / (float)a.R + a.eps);
    typename E::type *dst = (typename E::type *)a.slab + (page * PAGE_TOKENS + (t & (PAGE_TOKENS - 1))) * a.ldr;
    for (int r = threadIdx.x; r < a.R; r += THREADS) dst[r] = E::pack(X::load(x + r) * inv * a.w[r]);
}

// rotation in halves: number i of a vector with number i + dims / 2, by position * freq[i], cos and sin times gain; what lies behind dims stays
struct Rotation {
    const float *freq;
    int dims;
    float gain;
};
// one row's projections -> its normed query latent (cq; nullptr: not made), and (own) its normed latent and rotated key part into the page
struct LatentPrepArgs {
    const void *raw;       // [M][ld] T: query latent [Q8], latent [R8], key part [T8]
    int ld, M, Q, Q8, R, R8, T, T8;
    const float *q_norm, *c_norm;  // q_norm nullable: no weight
    float eps;
    Rotation rot;
    bool own;
    const int *pos, *row_seq, *table;
    int table_width, n_pages, n_seqs;
    void *cq;              // [M][ldc] T
    int ldc;
    void *slab;            // [n_pages][64][R8 + T8]
};
// the heads' vectors of every row, in place: row m, head h at q + m * ld + h * stride
struct RotateArgs {
    void *q;
    int ld, stride, H, M;
    Rotation rot;
    const int *pos;
};
template <class E>
__device__ __forceinline__ void rotate_pair(const typename E::type *u, const typename E::type *v, typename E::type *du, typename E::type *dv, float s, float c) {
    const float a = E::load(u), b = E::load(v);
    *du = E::pack(a * c - b * s), *dv = E::pack(b * c + a * s);
}
// row m's latent and key part into its page
template <class E, int THREADS>
__device__ __forceinline__ void latent_cache_row(const LatentPrepArgs &a, int m, float *red) {  // red: THREADS / 64 floats of LDS
    typedef typename E::type T;
    const T *c = (const T *)a.raw + (size_t)m * a.ld + a.Q8, *k = c + a.R8;
    const int t = a.pos[m];
    float ss = 0.0f;
    for (int i = threadIdx.x; i < a.R; i += THREADS) ss = fmaf(E::load(c + i), E::load(c + i), ss);
    ss = lanes_sum(ss);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    const size_t page = min((unsigned)a.table[(size_t)min(a.row_seq[m], a.n_seqs - 1) * a.table_width + min(t / PAGE_TOKENS, a.table_width - 1)], (unsigned)a.n_pages - 1u);
    T *row = (T *)a.slab + (page * PAGE_TOKENS + (t & (PAGE_TOKENS - 1))) * (a.R8 + a.T8), *rot = row + a.R8;
    const int half = a.rot.dims / 2;
    for (int i = threadIdx.x; i < half; i += THREADS) {
        float s, co;
        stack_sincos<sizeof(T) == 4>((float)t * a.rot.freq[i], s, co);
        rotate_pair<E>(k + i, k + half + i, rot + i, rot + half + i, s * a.rot.gain, co * a.rot.gain);
    }
    for (int i = 2 * half + threadIdx.x; i < a.T; i += THREADS) rot[i] = k[i];
    __syncthreads();
    float sum = red[0];
#pragma unroll
    for (int i = 1; i < THREADS / 64; ++i) sum += red[i];
    const float inv = 1.0f / sqrtf(sum / (float)a.R + a.eps);
    for (int i = threadIdx.x; i < a.R; i += THREADS) row[i] = E::pack(E::load(c + i) * inv * a.c_norm[i]);
}
// all heads of row m; a thread keeps one pair's angle for the heads it takes
template <class E, int THREADS>
__device__ __forceinline__ void rotate_row(const RotateArgs &a, int m) {
    typedef typename E::type T;
    const int half = a.rot.dims / 2;
    int lanes = 1;
    while (lanes < half && lanes < THREADS) lanes <<= 1;
    const float t = (float)a.pos[m];
    for (int i = threadIdx.x & (lanes - 1); i < half; i += lanes) {
        float s, c;
        stack_sincos<sizeof(T) == 4>(t * a.rot.freq[i], s, c);
        s *= a.rot.gain, c *= a.rot.gain;
        for (int h = threadIdx.x / lanes; h < a.H; h += THREADS / lanes) {
            T *p = (T *)a.q + (size_t)m * a.ld + h * a.stride + i;
            rotate_pair<E>(p, p + half, p, p + half, s, c);
        }
    }
}

// ---------------------------------------------------------------- the attention's key splits
// ws: sums [splits][M * H][ldr] fp32, then (maximum, sum of weights) [splits][M * H][2]; a split that saw no key has weight sum 0 and no sums
constexpr int MERGE_ROWS = 4, MERGE_LDR = 1024;
// what a head's sums are finished with: fp32 [H] a sink score in the denominator (nullable), [M][ldg] gate logits in the stack's dtype (nullable)
struct HeadFinish {
    const float *sink;
    const void *gate;
    int ldg;
};
template <bool F32>
__device__ __forceinline__ float head_gate(const HeadFinish &f, size_t row, int head) {
    if (!f.gate) return 1.0f;
    return 1.0f / (1.0f + expf(-(F32 ? ((const float *)f.gate)[row * f.ldg + head] : BF16::to_f32(((const u16 *)f.gate)[row * f.ldg + head]))));
}
// the sink's share of a denominator whose weights are relative to the exponent m (base 2)
__device__ __forceinline__ float head_sink2(const HeadFinish &f, int head, float m) { return f.sink ? __builtin_amdgcn_exp2f(f.sink[head] * STACK_LOG2E - m) : 0.0f; }
struct LatentMerge {
    const float *ws;
    int splits, M, H, ldr;
    HeadFinish finish;
};
// lane s: what split s of pair pr counts in the merged result (base 2 exponents; at most 64 splits)
__device__ __forceinline__ float latent_split_weight(const LatentMerge &a, size_t pr, int lane) {
    const size_t MH = (size_t)a.M * a.H;
    const float2 ml = lane < a.splits ? *(const float2 *)(a.ws + (size_t)a.splits * MH * a.ldr + (lane * MH + pr) * 2) : make_float2(-1e30f, 0.0f);
    const float m = wave_max(ml.y > 0.0f ? ml.x : -1e30f);
    const float f = ml.y > 0.0f ? __builtin_amdgcn_exp2f(ml.x - m) : 0.0f;
    return f * head_gate<false>(a.finish, pr / a.H, (int)(pr % a.H)) / (wave_sum(ml.y * f) + head_sink2(a.finish, (int)(pr % a.H), m));
}
// columns r .. r + 3 of the merged sums of pair pr, eight splits in flight; weight(s): a wave-uniform or per-thread read of split s's weight
template <class F>
__device__ __forceinline__ float4 latent_merge4(const LatentMerge &a, size_t pr, int r, F &&weight) {
    const size_t MH = (size_t)a.M * a.H;
    float4 acc = make_float4(0, 0, 0, 0);
    for (int s0 = 0; s0 < a.splits; s0 += 8) {
        float4 v[8];
        float w[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            const int s = min(s0 + u, a.splits - 1);
            w[u] = s0 + u < a.splits ? weight(s) : 0.0f;
            v[u] = *(const float4 *)(a.ws + (s * MH + pr) * a.ldr + r);
        }
#pragma unroll
        for (int u = 0; u < 8; ++u)
            if (w[u] > 0.0f) acc.x = fmaf(w[u], v[u].x, acc.x), acc.y = fmaf(w[u], v[u].y, acc.y), acc.z = fmaf(w[u], v[u].z, acc.z), acc.w = fmaf(w[u], v[u].w, acc.w);
    }
    return acc;
}

// ---------------------------------------------------------------- the row-wise Linear
enum RowsEpi {
    ROWS_STORE = 0,      // y[m][n] = T(v)
    ROWS_SCALE_F32 = 1,  // y[m][n] = v * scale, fp32 (logits; expert outputs, scale 1)
    ROWS_RELU2 = 2,      // y[m][n] = T(max(v, 0)^2)
    ROWS_SILU_MUL = 3,   // rows (2 i, 2 i + 1) = (gate_i, up_i): y[m][i] = T(silu(gate) * up)
    ROWS_SPLIT = 4,      // n < split: y[m][n] = T(v);  else y2[m][n - split] = v, fp32
    ROWS_RESIDUAL = 5,   // x[m][n] += post(v);  h[m][n] = T(next(x[m][n]))
    ROWS_CLIP_MUL = 6,   // rows (2 i, 2 i + 1) = (gate_i, up_i): y[m][i] = T(clipped_glu(gate, up))
    ROWS_XIELU = 7,      // y[m][n] = T(xielu(v))
    ROWS_GELU_MUL = 8,   // rows (2 i, 2 i + 1) = (gate_i, up_i), plus the bias: y[m][i] = T(gelu_tanh(gate) * up)
    ROWS_GELU_SIDE = 9,  // y[m][n] = T(gelu_tanh(v) * the row's token's side vector[n])
    ROWS_SOFTCAP = 10,   // y[m][n] = act_limit tanh(v * scale / act_limit), fp32 (capped logits)
};
// g sigmoid(alpha g) (u + 1) with g = min(gate, limit), u = clamp(up, -limit, limit)
__device__ __forceinline__ float clipped_glu(float gate, float up, float alpha, float limit) {
    const float g = fminf(gate, limit), u = fminf(fmaxf(up, -limit), limit);
    return g / (1.0f + expf(-alpha * g)) * (u + 1.0f);
}

struct RowsMat {      // one weight matrix with its operand and result
    const char *w;    // W16M tiles (bf16) or row-major fp32 [N][64 ceil(K / 64)]
    int N, K;
    const void *x;
    int ldx;          // elements
    void *y;
    int ldy;
};
// a vector per token id
struct TokenVectors {
    const u16 *table;  // bf16 [vocab][ld], the vector at `at`
    size_t ld, at;
    const int *ids;    // [M]
    int vocab;
};
__device__ __forceinline__ const u16 *token_vector(const TokenVectors &t, size_t m) { return t.table + (size_t)min(max(t.ids[m], 0), t.vocab - 1) * t.ld + t.at; }
constexpr int ROWS_LIST = 6;
struct RowsArgs {
    RowsMat m;
    int M;                 // rows of x (grouped: an upper bound for one expert's rows)
    // batched over blockIdx.y (heads): offsets per batch index
    size_t w_batch;        // bytes
    int x_batch, y_batch;  // elements
    // grouped over blockIdx.y (experts): active[y] = expert or -1; its rows are list[offset[e] .. offset[e + 1])
    const int *active, *offset, *list;
    bool gather;           // grouped: x row = list[position] (else x row = position); y row = position always
    RowsMat shared;        // blockIdx.y == batches - 1 when shared.w: all M rows, this matrix (the expert every token takes)
    const int *rows;       // ungrouped, nullable: x row of result row i
    RowsMat mats[ROWS_LIST];  // n_mats > 0: blockIdx.y picks one of these instead of m, each with its own sizes and operands
    int n_mats;
    const u16 *bias;       // ROWS_GELU_MUL: bf16 [N], nullable
    TokenVectors side;     // ROWS_GELU_SIDE
    int epi;
    float scale;
    float act_alpha, act_limit;  // ROWS_CLIP_MUL, ROWS_SOFTCAP; ROWS_XIELU: its two factors
    int split;
    float *y2;
    int ldy2;
    // ROWS_RESIDUAL
    float *res;            // [M][ld_res] residual stream
    int ld_res;
    PointNorm post, next;
    void *h;               // [M][ldh]
    int ldh;
    LatentMerge merge;     // merge.splits > 0 (batched over heads, bf16, at most MERGE_ROWS rows): x is merged from the attention's key splits on the way in
    bool x_norm;           // every row of x over its root mean square on the way in (fp32; with x_eps; ungrouped, bf16, at most 16 rows)
    float x_eps;
    // What rides along (M > 0) on blockIdx.y past the batches: it needs what this launch needs and would otherwise be launches of its own
    LatentAppend append;
    LatentPrepArgs cache;  // (the latent and key part only)
    RotateArgs rotate;     // (numbers of the same rows that this product does not read)
};
// batches: blockIdx.y extent (1 for a plain Linear; heads; active experts (+ 1 with a shared expert))
int rows_gemm_launch(int dtype, const RowsArgs &a, int batches, hipStream_t st);
// bytes of a packed [N, K] weight of the stack's dtype, and the repack from row-major bf16
size_t rows_weight_bytes(int dtype, int N, int K);

// ---------------------------------------------------------------- latent attention
// A pass holds runs of consecutive rows, one run per sequence; a workgroup takes 32 (token, head) pairs of ONE run.
struct RowRun {
    int row0, n_rows, seq, pos0;  // seq: row of the block table; pos0: position of row0 (single rows: not used, may be 0)
};
struct LatentAttnArgs {
    const void *q;         // [M][H][ldq]: queries in the latent space (W_uk^T q), ldq = row stride in elements
    const void *q_rot;     // nullable: [M][ld_rot], head h at h * (ldr - ldq): what meets the numbers of a cached row behind the latent
    int ldq, ld_rot;
    const void *slab;      // the layer's latent pages [n_pages][64][ldr]: the latent [ldq], and what scores read beside it
    const int *table;      // [n_seqs][table_width] page ids
    int table_width, n_pages, n_seqs;
    const int *pos;        // [M]
    const RowRun *runs;
    int n_runs, n_tiles;   // n_tiles = sum over the runs of latent_attn_tiles()
    bool single;           // every run is one row (a decode step): tile -> run without a search
    const int *row_seq;    // [M]
    int H, R, ldr, M;      // R: numbers of a row that scores read
    HeadFinish finish;
    int window;            // keys j with 0 <= i - j < window; <= 0: no limit
    float scale;
    int splits;            // > 1: fp32 partials in ws, merged by the combine launch (combine = false: left to the consumer)
    bool combine;
    float *ws;             // see LatentMerge
    void *out;             // [M][H][ldq] T: softmax-weighted latents
};
int latent_attn_launch(int dtype, const LatentAttnArgs &a, hipStream_t st);
int latent_attn_tiles(int n_rows, int H);
size_t latent_attn_ws_floats(int M, int H, int R, int splits);
int latent_append_launch(int dtype, const LatentAppend &a, hipStream_t st);

int latent_prep_launch(int dtype, const LatentPrepArgs &a, hipStream_t st);
int rotate_heads_launch(int dtype, const RotateArgs &a, hipStream_t st);

// ---------------------------------------------------------------- attention of long runs, keys and values spelled out (window_attn.hip)
constexpr int WINDOW_ATTN_MAX_DIM = 256;
struct WindowAttnArgs {
    const u16 *q, *kv;      // q [M][ld_q], head h at h * D8; kv [context rows][ld_kv]: keys of head h at h * D8, values at H * D8 + h * V8
    u16 *out;               // [M][ld_out], head h at h * V8
    int ld_q, ld_kv, ld_out, H, D8, V8, window;
    const u16 *q_rot, *k_rot;  // T8 > 0: a second part of queries (row stride ld_q, head h at h * T8) and of keys (row stride ld_krot, the same for all heads)
    int T8, ld_krot;
    HeadFinish finish;
    float scale;
    const RowRun *runs;     // the long runs; run r's context = positions [max(0, pos0 - window + 1), pos0 + n_rows), the runs' contexts concatenated in order
    int n_runs;
};
int window_attn_launch(const WindowAttnArgs &a, int n_tiles, hipStream_t st);  // n_tiles = sum of ceil(n_rows / 128)
int latent_gather_launch(const RowRun *runs, int n_runs, int n_ctx, int window, const int *table, int table_width, int n_seqs, int n_pages, const void *slab, int ldr,
                         void *out, int ld_out, hipStream_t st);

// ---------------------------------------------------------------- softmax attention over paged keys and values (page_attn.hip)
// A page of one layer holds, per key/value head, 64 keys and 64 values in matrix-core operand order: every operand load of a wave is one contiguous KiB.
//   key t (0 .. 63), dimension d:    two blocks of 32 keys, each [D16 / 8 chunks of 8 dimensions][32 keys][8]
//   value t, dimension d:            two blocks of 32 tokens, each [V32 / 32 blocks of 32 dimensions][2 halves of 16 tokens][2][32 dimensions][8 tokens], where the
//                                    8 tokens of (half s, h) are 16 s + 4 h + {0 .. 3, 8 .. 11}: the order in which the score product leaves its weights
// D16 = dim rounded up to 16, V32 = vdim rounded up to 32; what is never written stays zero.  fp32 stacks use the same order.
struct KvGeometry {
    int H, G, dim, vdim, D8, V8, D16, V32;  // D8, V8: head strides of activations
    __host__ __device__ size_t head_elems() const { return (size_t)PAGE_TOKENS * (D16 + V32); }
    __host__ __device__ size_t page_elems() const { return G * head_elems(); }
    __host__ __device__ int key(int t, int d) const { return (t >> 5) * 32 * D16 + ((d >> 3) * 32 + (t & 31)) * 8 + (d & 7); }
    __host__ __device__ int value(int t, int d) const {
        return PAGE_TOKENS * D16 + (t >> 5) * 32 * V32 + (d >> 5) * 1024 + ((t >> 4) & 1) * 512 + ((t >> 2) & 1) * 256 + (d & 31) * 8 + ((t & 3) | ((t >> 3) & 1) << 2);
    }
};
static inline KvGeometry kv_geometry(int H, int G, int dim, int vdim) {
    return {H, G, dim, vdim, (dim + 7) & ~7, (vdim + 7) & ~7, (dim + 15) & ~15, (vdim + 31) & ~31};
}
constexpr int PAGE_ATTN_MAX_DIM = 256;  // wider heads take the vector ALU (up to PAGE_ATTN_ROWS_DIM)
constexpr int PAGE_ATTN_ROWS_DIM = 1024;

struct PageTable {  // where a sequence's pages are
    const int *table;
    int table_width, n_pages, n_seqs;
};
__device__ __forceinline__ int page_of(const PageTable &p, int seq, int t) {
    const int j = min(t / PAGE_TOKENS, p.table_width - 1);
    return (int)min((unsigned)p.table[(size_t)min(seq, p.n_seqs - 1) * p.table_width + j], (unsigned)p.n_pages - 1u);
}

// raw projections -> normed and rotated queries (in place), keys and values of the pass's rows into their pages
struct KvPrepArgs {
    void *raw;              // [M][ld] T: q [H][D8], k [G][D8], v [G][V8] (own), gate
    int ld, M;
    const u16 *bias;        // bf16, same order; nullable
    KvGeometry geo;
    bool own, value_norm;   // own: the layer has keys and values of its own
    const float *q_norm, *k_norm;
    bool row_norm;          // the norms run over all heads of a row at once, weights [heads][D8], and values are the keys in front of their norm (no v in raw); no rotation
    float eps;
    const float *freq;
    int rot_dims;
    float rot_gain;
    const int *pos, *row_seq;
    PageTable pages;
    void *slab;
};
int kv_prep_launch(int dtype, const KvPrepArgs &a, hipStream_t st);

struct PageAttnArgs {
    const void *q;          // [M][ldq] T, head h at h * D8
    int ldq;
    const void *slab;
    PageTable pages;
    KvGeometry geo;
    const int *pos, *row_seq;
    const RowRun *runs;
    int n_runs, n_tiles, M;
    bool single;            // every run is one row
    int window;             // keys j with 0 <= i - j < window; <= 0: no limit
    int chunk;              // > 0: keys of the query's own chunk (i / chunk = j / chunk) instead
    const float *distance;  // fp32 [H][far + 1], nullable: added to the scaled score of a key min(i - j, far) tokens back
    int far;
    const float *head_sink; // fp32 [H], nullable: one more score in the denominator (then sink is 0)
    float out_scale;        // factor on every head's output
    float scale, sink;      // score = scale q . k (+ distance); sink: what the softmax's denominator has besides the keys, as the weight of one more score of 0
    const void *gate;       // [M][ldg] T logits per head, nullable: every head's output times their sigmoid
    const u16 *gate_bias;   // bf16 [H], nullable
    int ldg;
    int splits;
    float *ws;              // see LatentMerge (ldr = V32)
    void *out;              // [M][ld_out] T, head h at h * V8
    int ld_out;
};
int page_attn_tiles(int n_rows, const KvGeometry &g);       // of the short form
int page_attn_long_tiles(int n_rows, const KvGeometry &g);  // of the long form
size_t page_attn_ws_floats(int M, const KvGeometry &g, int splits);
bool page_attn_mfma(int dtype, const KvGeometry &g);        // matrix-core forms exist for this shape (else: one launch for any rows)
int page_attn_launch(int dtype, const PageAttnArgs &a, hipStream_t st);
int page_attn_long_launch(const PageAttnArgs &a, hipStream_t st);

// ---------------------------------------------------------------- generalised delta rule (delta_rule.hip)
constexpr int DELTA_MAX_DIM = 256, DELTA_MAX_RANK = 1024;
constexpr float DELTA_MAX_DECAY = 2.0f;
struct DeltaArgs {
    const void *raw;        // [M][ld] T: r, k, v, gate, rate [H][D8] each, then the decay's low-rank input [rank]
    int ld, M, H, D, D8, rank, R8;
    const u16 *bias;        // bf16, same order; nullable
    const u16 *w_decay;     // bf16 [H * D][R8]
    const float *decay_bias, *o_norm;
    float decay_scale, unit_eps, eps;
    const int *pos, *row_seq, *slots;
    int n_seqs, n_slots;
    const RowRun *runs;
    int n_runs;
    float *state;           // [n_slots][slot_floats], of which [H][D][D] (key channel, value column)
    size_t slot_floats;
    float *ws, *o;          // chunk form: delta_ws_floats(); outputs [M][H][D8] in front of norm and gate
    int chunk_lo, chunk_hi; // (set by the launcher: the chunks of one segment)
    void *out;              // [M][ld_out] T, head h at h * D8
    int ld_out;
};
int delta_step_launch(int dtype, const DeltaArgs &a, hipStream_t st);  // token by token
// runs of many tokens, covering rows [row0, row0 + rows); chunks: sum of delta_chunks() over the runs
int delta_chunks_launch(int dtype, const DeltaArgs &a, int chunks, int row0, int rows, hipStream_t st);
int delta_chunks(int n_rows);
size_t delta_ws_floats(int chunks, int H, int D);
int delta_launches(int chunks, int H, int D);

// causal convolutions over time: taps at most, rows of a run per tile (conv_tiles())
constexpr int CONV_MAX_TAPS = 16, CONV_ROWS = 16;

// ---------------------------------------------------------------- gated delta rule (gated_delta.hip)
constexpr int GATED_MAX_DIM = 256;
struct GatedDeltaArgs {
    const void *raw;        // [M][ld] T: q, k [G][D8] each, v, gate [H][V8] each, step size, decay [H8] each
    int ld, M, H, G, D, D8, V, V8, H8;
    const float *conv;      // fp32 [taps][ldw] over the channels of q, k, v; the last tap reads the token itself
    int taps, ldw;
    const float *decay_rate, *decay_bias, *o_norm;  // fp32 [H], [H], [V]
    float scale, unit_eps, eps;
    const int *pos, *row_seq, *slots;
    int n_seqs, n_slots;
    const RowRun *runs;
    int n_runs;
    float *state;           // [n_slots][slot_floats]: [H][D][V], then (at ring) [taps][channels] the last inputs of the convolution, position p at p mod taps
    size_t slot_floats, ring;
    void *mixed;            // [M][channels] T: convolved and activated q, k, v; nullptr (step form, every run one row): taken on the way
    float *ws, *o;          // chunk form: gated_delta_ws_floats(); outputs [M][H][V8] in front of norm and gate (also heads of more than 256 columns)
    void *out;              // [M][ld_out] T, head h at h * V8
    int ld_out;
};
__host__ __device__ static inline int gated_delta_channels(int H, int G, int D8, int V8) { return 2 * G * D8 + H * V8; }
int gated_delta_conv_launch(int dtype, const GatedDeltaArgs &a, int tiles, hipStream_t st);  // all runs; tiles: sum of conv_tiles()
int gated_delta_step_launch(int dtype, const GatedDeltaArgs &a, int row0, int rows, hipStream_t st);
int gated_delta_chunks_launch(int dtype, const GatedDeltaArgs &a, int chunks, int row0, int rows, hipStream_t st);
size_t gated_delta_ws_floats(int chunks, int H, int D);
int gated_delta_chunk_launches(int chunks, int H, int D);

// ---------------------------------------------------------------- time mixing with a decaying matrix state (time_mix.hip)
constexpr int TIME_MIX_MAX_DIM = 256, TIME_MIX_MAX_RANK = 1024, TIME_MIXES = 5;
struct TimeMixArgs {
    const void *r, *k, *v, *gate;  // [M][ld] T each, head h at h * D8
    const void *low;               // [M][ld_low] T: the decay's low-rank input
    int ld, ld_low, M, H, D, D8, rank, R8;
    const u16 *w_decay;            // bf16 [H * D][R8]
    const float *decay_bias, *bonus, *o_norm;  // fp32 [H * D] each
    float eps, out_scale;
    const int *pos, *row_seq, *slots;
    int n_seqs, n_slots;
    const RowRun *runs;
    int n_runs;
    float *state;                  // [n_slots][slot_floats], of which [H][D][D] (key channel, value column)
    size_t slot_floats;
    float *ws, *o;                 // chunk form
    void *out;                     // [M][ld_out] T, head h at h * D8
    int ld_out;
};
int time_mix_step_launch(int dtype, const TimeMixArgs &a, int row0, int rows, hipStream_t st);
int time_mix_chunks_launch(int dtype, const TimeMixArgs &a, int chunks, int row0, int rows, hipStream_t st);
size_t time_mix_ws_floats(int chunks, int H, int D);
int time_mix_chunk_launches(int chunks, int H, int D);

// every head's output over its root mean square, times w and the sigmoid (or silu) of its gate (head_out.hip)
struct HeadOutArgs {
    const float *o;         // [M][H][D8]
    const float *den;       // [M][H], what o is divided by first; nullable
    const void *gate;       // [M][ldg] T logits, head h at h * D8
    const u16 *gate_bias;   // bf16 [H * D8]; nullable
    int ldg, H, D, D8;
    const float *w;         // [H][D]
    float eps;
    void *out;              // [M][ld_out] T, head h at h * D8
    int ld_out;
    bool shared_w, silu;    // w is [D], the same for all heads; gates are z sigmoid(z)
    float scale;
};
constexpr int HEAD_OUT_MAX_DIM = 2048;
int head_out_launch(int dtype, const HeadOutArgs &a, int row0, int rows, hipStream_t st);

// ---------------------------------------------------------------- recurrences whose gates read the current token only
struct RecurrentArgs {
    const void *raw;        // [M][ld] T, the mixer's projections
    int ld, M;
    const int *pos, *row_seq, *slots;
    int n_seqs, n_slots;
    const RowRun *runs;
    int n_runs;
    float *state;           // [n_slots][slot_floats]
    size_t slot_floats;
    float *ws;              // chunk forms
};
__device__ __forceinline__ float *recurrent_state(const RecurrentArgs &a, const RowRun &run) {
    return a.state + min((unsigned)a.slots[min(a.row_seq[run.row0], a.n_seqs - 1)], (unsigned)a.n_slots - 1u) * a.slot_floats;
}
// chunk i of the runs in pieces of `size` rows
struct RowChunk {
    int run, row0, n, pos;  // pos: places of the run in front of it
};
__device__ __forceinline__ RowChunk row_chunk(const RowRun *runs, int n_runs, int i, int size) {
    int r = 0;
    for (;;) {
        const int n = (runs[r].n_rows + size - 1) / size;
        if (i < n || r + 1 >= n_runs) break;
        i -= n, ++r;
    }
    return {r, runs[r].row0 + size * i, min(size, runs[r].n_rows - size * i), size * i};
}

// minGRU (mingru.hip): S_t = (1 - z) S_(t-1) + z candidate per channel; out = S_t silu(gate)
struct MingruArgs {
    RecurrentArgs r;        // raw: z, candidate, gate [D8] each
    const u16 *bias;        // bf16, same order; nullable
    int D, D8;
    void *out;              // [M][ld_out] T
    int ld_out;
};
int mingru_step_launch(int dtype, const MingruArgs &a, hipStream_t st);                 // token by token
int mingru_chunks_launch(int dtype, const MingruArgs &a, int chunks, hipStream_t st);  // runs of many tokens
int mingru_chunks(int n_rows);
size_t mingru_ws_floats(int chunks, int D);

// mLSTM (mlstm.hip): a matrix memory per head with exponential gates
struct MlstmArgs {
    RecurrentArgs r;        // raw: q, k [H][D8] each, v, output gate [H][V8] each, input gate, forget gate [H8] each
    const float *gate_bias; // [2][H]: input, forget
    int H, D, D8, V, V8, H8;
    float scale, cap, den_eps;
    float *o, *den;         // [M][H][V8] sums, [M][H] what they are divided by
};
constexpr int MLSTM_MAX_DIM = 1024, MLSTM_CHUNK_MAX_DIM = 512;
size_t mlstm_state_floats(int H, int D, int V);
int mlstm_step_launch(int dtype, const MlstmArgs &a, hipStream_t st);       // token by token
int mlstm_chunks_launch(const MlstmArgs &a, int chunks, hipStream_t st);   // runs of many tokens (bf16)
int mlstm_chunks(int n_rows);
size_t mlstm_ws_floats(int chunks, int H, int D, int V);

// ---------------------------------------------------------------- x += post(y); h = next(x) with norms that need the whole row (row_update.hip)
struct StackNorm {
    const float *w, *b;
    float param;
    int kind;
};
constexpr int ROW_UPDATE_MAX_WIDTH = 32768;
// mixes of every row with its predecessor in the sequence: out[s][m] = x_m + (x_(m-1) - x_m) mu[s], s < TIME_MIXES; the state carries the last row
struct TokenMixArgs {
    const float *mu;        // fp32 [TIME_MIXES][ldmu]; nullptr: none
    int ldmu;
    float *state;           // [n_slots][slot_floats], of which [W rounded up to 4]
    size_t slot_floats;
    const int *pos, *row_seq, *slots;
    int n_seqs, n_slots;
    const RowRun *runs;
    int n_runs;
    void *out;              // [TIME_MIXES][M][ldo] T
    int ldo;
};
struct RowUpdateArgs {
    const void *y;          // [M][ldy] (nullptr: x stays as it is, h = next(x)); experts: [M * top][ldy] by position
    bool y32;               // y is fp32 (else bf16)
    int ldy;
    const u16 *bias;        // bf16 [W] added to y; nullable
    const int *place;       // experts (nullable): y of row m = sum over its slots s of weight[m * top + s] * y[place[m * top + s]]
    const float *weight;    // nullable: 1 / top each
    int top;
    StackNorm post, next;
    bool after;             // the norm runs over the sum: x = post(alpha x + y)
    float alpha;
    float *x;               // [M][ldx]
    int ldx;
    void *h;                // [M][ldh] T
    int ldh, M, W;
    // nullable: the rows choose their experts on the way, by the router's logits of next(x) (fp32); lists as k_route makes them, without tiles
    const struct RouteLayer *route;
    int experts;
    const u16 *router;      // bf16 [experts][W rounded up to 8], zeros past W
    int *arrived;           // one int, zero before and after
    TokenMixArgs mix;       // of the new x; only where every run is one row
};
int row_update_launch(int dtype, const RowUpdateArgs &a, hipStream_t st);
int token_mix_launch(int dtype, const TokenMixArgs &a, const float *x, int ldx, int M, int W, hipStream_t st);  // any runs

// ---------------------------------------------------------------- residual streams (stream_update.hip)
// x_t <- sum_s mix[s][t] x_s + out[t] y;  h = next(sum_s in[s] x_s), and the causal convolution over time in front of a mixer: h + conv(h)
constexpr int STREAMS_MAX = 16;
struct StackEmbed {
    const int *ids;         // nullptr: the streams are in memory already
    const u16 *table, *bigram, *positions;  // bf16 [vocab][W]; [buckets + 1][W], [max_positions][W], nullable
    float scale;
    int vocab, buckets, max_positions;
    long long mul_prev, mul_cur;
    float *prev;            // [n_slots][slot_floats]: the sequences' previous tokens (as integers)
};
struct ConvArgs {
    const float *w;         // [taps][ldw], tap taps - 1 reads the row itself; nullptr: none
    int taps, ldw;
    float *state;           // [n_slots][slot_floats], of which [taps - 1][W rounded up to 4]: the last inputs, oldest first
    const int *pos, *row_seq, *slots;
    int n_seqs, n_slots;
    size_t slot_floats;
    const RowRun *runs;
    int n_runs;
};
struct StreamUpdateArgs {
    StackEmbed embed;
    const void *y;          // [M][ldy]; nullptr: the streams stay as they are
    bool y32;               // y is fp32 (else bf16)
    int ldy;
    const float *out, *mix; // [S], [S][S] (from, to)
    float *x;               // [M][S][ldx]
    int ldx, S;
    const float *in;        // [S]; nullptr: the streams' sum
    StackNorm next;
    ConvArgs conv;          // single: taken here (conv.w may be nullptr); else only its slots are used, and conv_launch follows
    bool single;            // every run is one row
    void *h;                // [M][ldh] T
    int ldh, M, W;
};
int stream_update_launch(int dtype, const StreamUpdateArgs &a, hipStream_t st);
// h = hc + conv(hc) over runs of several rows; carries the state
int conv_launch(int dtype, const ConvArgs &a, const void *hc, void *h, int ldh, int W, int tiles, hipStream_t st);
int conv_tiles(int n_rows);
// out[m][W] = sum of the streams
int stream_sum_launch(const float *x, int ldx, int S, float *out, int M, int W, hipStream_t st);
