// mingru.hip -- minGRU (PIE_MIXER_MINGRU): per channel S_t = (1 - z_t) S_(t-1) + z_t c_t in fp32, z = sigmoid(.), c = u + 1/2 where u >= 0 and sigmoid(u) where u < 0;
// out = S_t silu(gate).  The gates read the current token only, so a run of tokens is a linear recurrence with known factors.
//
// Step form (decoded tokens, short runs): a thread walks the run's tokens for two channels.
// Chunk form: pieces of 64 tokens.  One launch makes every piece's (product of the factors, state from zero), a second chains the pieces (and carries the
// sequence's state), a third walks every piece again from the state in front of it and writes the outputs.
#include "stack_types.hpp"

namespace {

constexpr int MG = 64;  // tokens of a piece

struct MgPair {
    float x, y;
};
template <class T>
__device__ __forceinline__ MgPair mg_pair(const T *p) {
    if constexpr (sizeof(T) == 4) return {((const float2 *)p)->x, ((const float2 *)p)->y};
    else {
        const u32 w = *(const u32 *)p;
        return {lo_f32<BF16>(w), hi_f32<BF16>(w)};
    }
}
__device__ __forceinline__ MgPair mg_bias(const MingruArgs &a, int at) {
    if (!a.bias) return {0.0f, 0.0f};
    const u32 w = *(const u32 *)(a.bias + at);
    return {lo_f32<BF16>(w), hi_f32<BF16>(w)};
}
// (keep, add): S <- keep S + add
template <bool F32>
__device__ __forceinline__ MgPair mg_gate(float z, float u) {
    const float g = stack_sigmoid<F32>(z), c = u >= 0.0f ? u + 0.5f : stack_sigmoid<F32>(u);
    return {1.0f - g, g * c};
}
template <class E>
__device__ __forceinline__ void mg_store(const MingruArgs &a, size_t m, int d, float sx, float sy, const MgPair &g, const MgPair &bg) {
    typedef typename E::type T;
    constexpr bool F32 = sizeof(T) == 4;
    const float gx = g.x + bg.x, gy = g.y + bg.y;
    const float x = sx * gx * stack_sigmoid<F32>(gx), y = d + 1 < a.D ? sy * gy * stack_sigmoid<F32>(gy) : 0.0f;
    T *out = (T *)a.out + m * a.ld_out + d;
    if constexpr (F32) *(float2 *)out = make_float2(x, y);
    else *(u32 *)out = pack2<BF16>(x, y);
}

constexpr int MG_AHEAD = 16;  // tokens in flight

// walks rows [row0, row0 + n) from (sx, sy); OUT: writes the outputs; else accumulates the factors' products
template <class E, bool OUT>
__device__ __forceinline__ void mg_walk(const MingruArgs &a, int row0, int n, int d, float &sx, float &sy, float &px, float &py) {
    typedef typename E::type T;
    constexpr bool F32 = sizeof(T) == 4;
    const MgPair bz = mg_bias(a, d), bu = mg_bias(a, a.D8 + d), bg = mg_bias(a, 2 * a.D8 + d);
    for (int t0 = 0; t0 < n; t0 += MG_AHEAD) {
        MgPair z[MG_AHEAD], u[MG_AHEAD], g[MG_AHEAD];
#pragma unroll
        for (int t = 0; t < MG_AHEAD; ++t) {
            const T *x = (const T *)a.r.raw + (size_t)(row0 + min(t0 + t, n - 1)) * a.r.ld + d;
            z[t] = mg_pair(x), u[t] = mg_pair(x + a.D8);
            if constexpr (OUT) g[t] = mg_pair(x + 2 * a.D8);
        }
#pragma unroll
        for (int t = 0; t < MG_AHEAD; ++t) {
            if (t0 + t >= n) continue;
            const MgPair p = mg_gate<F32>(z[t].x + bz.x, u[t].x + bu.x), q = mg_gate<F32>(z[t].y + bz.y, u[t].y + bu.y);
            sx = fmaf(p.x, sx, p.y), sy = fmaf(q.x, sy, q.y);
            if constexpr (OUT) mg_store<E>(a, row0 + t0 + t, d, sx, sy, g[t], bg);
            else px *= p.x, py *= q.x;
        }
    }
}

template <class E>
__global__ void __launch_bounds__(64) k_mingru_step(const MingruArgs a) {
    const int d = 2 * (blockIdx.x * 64 + threadIdx.x);
    const RowRun run = a.r.runs[blockIdx.y];
    if (d >= a.D) return;
    float *state = recurrent_state(a.r, run) + d;
    float sx = 0.0f, sy = 0.0f, px, py;
    if (a.r.pos[run.row0] != 0) sx = state[0], sy = state[1];  // (the state holds an even number of channels)
    mg_walk<E, true>(a, run.row0, run.n_rows, d, sx, sy, px, py);
    *(float2 *)state = make_float2(sx, sy);
}

// ws: [chunks][2][D8]: products, then states from zero; the chain leaves the state in front of every piece in the first
template <class E>
__global__ void __launch_bounds__(64) k_mingru_pieces(const MingruArgs a) {
    const int d = 2 * (blockIdx.x * 64 + threadIdx.x);
    const RowChunk c = row_chunk(a.r.runs, a.r.n_runs, blockIdx.y, MG);
    if (d >= a.D || c.n <= 0) return;
    float sx = 0.0f, sy = 0.0f, px = 1.0f, py = 1.0f;
    mg_walk<E, false>(a, c.row0, c.n, d, sx, sy, px, py);
    float *ws = a.r.ws + (size_t)blockIdx.y * 2 * a.D8 + d;
    *(float2 *)ws = make_float2(px, py);
    *(float2 *)(ws + a.D8) = make_float2(sx, sy);
}
__global__ void __launch_bounds__(64) k_mingru_chain(const MingruArgs a) {
    const int d = blockIdx.x * 64 + threadIdx.x;
    if (d >= a.D) return;
    int chunk0 = 0;
    for (int r = 0; r < (int)blockIdx.y; ++r) chunk0 += (a.r.runs[r].n_rows + MG - 1) / MG;
    const RowRun run = a.r.runs[blockIdx.y];
    const int n = (run.n_rows + MG - 1) / MG;
    float *state = recurrent_state(a.r, run) + d, S = a.r.pos[run.row0] == 0 ? 0.0f : *state;
    float *ws = a.r.ws + (size_t)chunk0 * 2 * a.D8 + d;
    constexpr int U = 16;
    for (int c0 = 0; c0 < n; c0 += U) {
        float p[U], s[U];
#pragma unroll
        for (int i = 0; i < U; ++i) {
            const size_t at = (size_t)min(c0 + i, n - 1) * 2 * a.D8;
            p[i] = ws[at], s[i] = ws[at + a.D8];
        }
#pragma unroll
        for (int i = 0; i < U; ++i) {
            if (c0 + i >= n) break;
            ws[(size_t)(c0 + i) * 2 * a.D8] = S;
            S = fmaf(p[i], S, s[i]);
        }
    }
    *state = S;
}
template <class E>
__global__ void __launch_bounds__(64) k_mingru_out(const MingruArgs a) {
    const int d = 2 * (blockIdx.x * 64 + threadIdx.x);
    const RowChunk c = row_chunk(a.r.runs, a.r.n_runs, blockIdx.y, MG);
    if (d >= a.D || c.n <= 0) return;
    const float2 s = *(const float2 *)(a.r.ws + (size_t)blockIdx.y * 2 * a.D8 + d);
    float sx = s.x, sy = s.y, px, py;
    mg_walk<E, true>(a, c.row0, c.n, d, sx, sy, px, py);
}

int mingru_check(const MingruArgs &a) {
    PIE_REQUIRE(a.D > 0 && a.D8 % 8 == 0 && a.r.ld % 2 == 0 && a.ld_out % 2 == 0 && a.r.slot_floats % 2 == 0, PIE_E_SHAPE, "minGRU: bad sizes");
    PIE_REQUIRE(a.r.slots && a.r.state && a.r.n_slots > 0 && a.r.n_runs <= 65535, PIE_E_ARG, "minGRU: no state slots");
    return PIE_OK;
}

template <class E>
int mingru_chunks_go(const MingruArgs &a, int chunks, hipStream_t st) {
    const unsigned x = (unsigned)((a.D + 127) / 128);
    hipLaunchKernelGGL(k_mingru_pieces<E>, dim3(x, (unsigned)chunks), dim3(64), 0, st, a);
    PIE_LAUNCH_CHECK();
    hipLaunchKernelGGL(k_mingru_chain, dim3((unsigned)((a.D + 63) / 64), (unsigned)a.r.n_runs), dim3(64), 0, st, a);
    PIE_LAUNCH_CHECK();
    hipLaunchKernelGGL(k_mingru_out<E>, dim3(x, (unsigned)chunks), dim3(64), 0, st, a);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

}  // namespace

int mingru_chunks(int n_rows) { return (n_rows + MG - 1) / MG; }
size_t mingru_ws_floats(int chunks, int D) { return (size_t)chunks * 2 * ((D + 7) & ~7); }

int mingru_step_launch(int dtype, const MingruArgs &a, hipStream_t st) {
    if (a.r.n_runs <= 0) return PIE_OK;
    if (const int rc = mingru_check(a)) return rc;
    const dim3 grid((unsigned)((a.D + 127) / 128), (unsigned)a.r.n_runs);
    if (dtype == PIE_F32) hipLaunchKernelGGL(k_mingru_step<ElemF32>, grid, dim3(64), 0, st, a);
    else hipLaunchKernelGGL(k_mingru_step<ElemBF16>, grid, dim3(64), 0, st, a);
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

int mingru_chunks_launch(int dtype, const MingruArgs &a, int chunks, hipStream_t st) {
    if (a.r.n_runs <= 0) return PIE_OK;
    if (const int rc = mingru_check(a)) return rc;
    PIE_REQUIRE(a.r.ws && chunks > 0 && chunks <= 65535, PIE_E_ARG, "minGRU: the chunk form needs its workspace");
    return dtype == PIE_F32 ? mingru_chunks_go<ElemF32>(a, chunks, st) : mingru_chunks_go<ElemBF16>(a, chunks, st);
}
