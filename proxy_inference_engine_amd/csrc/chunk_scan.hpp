// chunk_scan.hpp -- the walk over the chunks of a recurrence with a matrix state per head, S [key channel][value column] in fp32, 16 tokens at a time on the fp32 matrix
// cores.  Everything but S has been made beforehand (k_*_prep of delta_rule.hip, gated_delta.hip, time_mix.hip), in matrix operand order, per chunk and head:
//   SCAN_DELTA   P = U S + X V,  O = R S + Y V + Z P,  S <- w S + K V + M P      (what a token removes, P, and what it writes, V, go different ways)
//   SCAN_GATED   P = U S + X V,  O = R S + Y P,        S <- w S + K P            (P: what a token writes, which is its value minus what the state holds for its key)
//   SCAN_LINEAR                  O = R S + Y V,        S <- w S + K V
// U, R [16 tokens][channels], K, M [channels][16 tokens], X, Y, Z [16][16], w one factor per channel; V the chunk's values.
//
// One workgroup per head and 16 value columns; its four waves split the key channels of S, which stays in accumulators and is its own B operand.  The operands' order in
// the workspace: U, R, K, M as far as the kind has them ([blocks of 16 channels][64 lanes][4] each), X, Y, Z likewise ([64 lanes][4]), w [16 blocks].
#pragma once
#include <algorithm>

#include "stack_types.hpp"

typedef __attribute__((ext_vector_type(4))) float dr_f32x4;
typedef __attribute__((ext_vector_type(8))) __bf16 dr_bf16x8;

namespace {

enum { SCAN_DELTA = 0, SCAN_GATED = 1, SCAN_LINEAR = 2 };
constexpr int DC = 16;  // tokens of a chunk
constexpr size_t SCAN_SEGMENT_BYTES = 96u << 20;

__host__ __device__ constexpr int scan_ops(int kind) { return kind == SCAN_DELTA ? 4 : kind == SCAN_GATED ? 3 : 2; }
__host__ __device__ constexpr int scan_mats(int kind) { return kind == SCAN_DELTA ? 3 : kind == SCAN_GATED ? 2 : 1; }
__host__ __device__ __forceinline__ int dr_blocks(int D) { return (D + 15) / 16; }
__host__ __device__ __forceinline__ size_t scan_chunk_floats(int kind, int D) { return (size_t)dr_blocks(D) * (scan_ops(kind) * 256 + 16) + scan_mats(kind) * 256; }

__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }  // (loads and stores stay in flight)
__device__ __forceinline__ dr_f32x4 dr_mfma(float a, float b, const dr_f32x4 &c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

struct ScanArgs {
    const void *v;          // [M][ld] T: head h's values at h * V8
    const u16 *bias;        // bf16, added to the values; nullable
    int ld, H, D, V, V8;
    const int *pos, *row_seq, *slots;
    int n_seqs, n_slots;
    const RowRun *runs;
    int n_runs;
    float *state;           // [n_slots][slot_floats], of which [H][D][V]
    size_t slot_floats;
    const float *ws;
    float *o;               // [M][H][V8]
    int chunk_lo, chunk_hi; // the chunks of this launch
};

struct ScanChunk {
    int row0, n;  // rows [row0, row0 + n)
};
__device__ __forceinline__ ScanChunk scan_chunk(const RowRun *runs, int n_runs, int i) {
    int r = 0;
    for (;;) {
        const int n = (runs[r].n_rows + DC - 1) / DC;
        if (i < n || r + 1 >= n_runs) break;
        i -= n, ++r;
    }
    return {runs[r].row0 + DC * i, min(DC, runs[r].n_rows - DC * i)};
}

// column n16 of (I + B)^-1 for a strictly lower B whose transpose is at b ([16][LM]), by forward substitution; lane n16 of every quarter of the wave
template <int LM>
__device__ __forceinline__ void scan_inverse(const float *b, int n16, float (&tc)[DC]) {
#pragma unroll
    for (int t = 0; t < DC; ++t) tc[t] = t == n16 ? 1.0f : 0.0f;
#pragma unroll
    for (int i = 0; i < DC - 1; ++i)
#pragma unroll
        for (int t4 = i / 4; t4 < DC / 4; ++t4) {
            const dr_f32x4 col = *(const dr_f32x4 *)(b + i * LM + 4 * t4);
#pragma unroll
            for (int k = 0; k < 4; ++k)
                if (4 * t4 + k > i) tc[4 * t4 + k] = fmaf(-col[k], tc[i], tc[4 * t4 + k]);
        }
}

// A chunk's operands are further away than a chunk takes, so they travel through LDS by DMA, RING - 1 chunks ahead; every wave fetches, waits for and reads
// only its own.
template <class E, int NB, int KIND>
struct ScanLds {
    static constexpr int NOP = scan_ops(KIND), PIECES = NOP * NB + 2;
    static constexpr int DW = 16 * sizeof(typename E::type) / 4, VI = 16 * DW / 64;  // dwords of a token's 16 values; DMA instructions for the chunk's
    static constexpr int OPS = PIECES + VI;                                          // DMA instructions per wave and chunk
    static constexpr int WAVE = PIECES * 1024 + VI * 256, SLOT = 4 * WAVE;
    static constexpr int PB = NB <= 3 ? 2 : 1;  // buffers of the exchanges between the waves
    static constexpr int RING = 5 * SLOT <= 128 * 1024 ? 5 : 3 * SLOT <= 136 * 1024 ? 3 : 2;
};
template <class E, int NB, int KIND>
__global__ void __launch_bounds__(256, 1) k_scan(const ScanArgs a) {
    typedef typename E::type T;
    typedef ScanLds<E, NB, KIND> L;
    constexpr int NOP = L::NOP, OR = KIND == SCAN_LINEAR ? 0 : 1, OK = OR + 1;  // U, R, K, M: operands 0, OR, OK, 3
    __shared__ __attribute__((aligned(1024))) char s_ring[L::RING * L::SLOT];
    __shared__ dr_f32x4 s_p[KIND == SCAN_LINEAR ? 1 : L::PB][4][64], s_o[L::PB][4][64];
    const int D = a.D, V = a.V, nblk = dr_blocks(D), lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), n16 = lane & 15, q = lane >> 4;
    const int head = (int)blockIdx.x % a.H, cb = (int)blockIdx.x / a.H, col = 16 * cb + n16;  // (head fastest: the column blocks of a head share an L2 where H is a multiple of 8)
    const RowRun run = a.runs[blockIdx.y];
    int chunk0 = 0;
    for (int r = 0; r < (int)blockIdx.y; ++r) chunk0 += (a.runs[r].n_rows + DC - 1) / DC;
    const int c_lo = max(a.chunk_lo - chunk0, 0), c_hi = min(a.chunk_hi - chunk0, (run.n_rows + DC - 1) / DC);  // this launch's chunks of the run
    if (c_lo >= c_hi) return;
    const size_t slot = min((unsigned)a.slots[min(a.row_seq[run.row0], a.n_seqs - 1)], (unsigned)a.n_slots - 1u);
    float *state = a.state + slot * a.slot_floats + (size_t)head * D * V;
    const bool fresh = c_lo == 0 && a.pos[run.row0] == 0;
    dr_f32x4 S[NB];  // S[16 b + 4 q + i][col]
#pragma unroll
    for (int j = 0; j < NB; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int d = 16 * (wave * NB + j) + 4 * q + i;
            S[j][i] = !fresh && d < D && col < V ? state[(size_t)d * V + col] : 0.0f;
        }
    const size_t per = scan_chunk_floats(KIND, D);
    const float *ws = a.ws + ((ptrdiff_t)(chunk0 - a.chunk_lo) * a.H + head) * (ptrdiff_t)per;  // chunk c of the run at c * H * per
    const char *vp = (const char *)((const T *)a.v + (size_t)run.row0 * a.ld + head * a.V8 + 16 * cb);
    const float vbias = a.bias ? BF16::to_f32(a.bias[head * a.V8 + min(col, V - 1)]) : 0.0f;
    const unsigned lds0 = (unsigned)(size_t)(__attribute__((address_space(3))) void *)s_ring + (unsigned)(wave * L::WAVE);
    auto scalar = [&](const void *p) {
        const unsigned long long v = (unsigned long long)(uintptr_t)p;
        return (unsigned long long)(unsigned)__builtin_amdgcn_readfirstlane((int)(unsigned)v) | ((unsigned long long)(unsigned)__builtin_amdgcn_readfirstlane((int)(unsigned)(v >> 32)) << 32);
    };
    auto fetch = [&](int cc, int at) {  // chunk cc (behind the end: the last one again, the waits count instructions) into ring slot `at`
        const int c = min(cc, c_hi - 1);
        const unsigned dst0 = lds0 + (unsigned)(at * L::SLOT);
        const unsigned long long base = scalar(ws + (size_t)c * a.H * per);
        auto piece = [&](unsigned byte, unsigned dst) {
            unsigned keep;
            asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %3\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, %2\n\ts_mov_b32 m0, %0"
                         : "=&s"(keep)
                         : "v"(byte + (unsigned)lane * 16u), "s"(base), "s"(dst)
                         : "memory");
        };
#pragma unroll
        for (int j = 0; j < NB; ++j) {
            const int b = min(wave * NB + j, nblk - 1);  // (blocks past the end meet channels that stay zero)
#pragma unroll
            for (int k = 0; k < NOP; ++k) piece((unsigned)(k * nblk + b) * 1024u, dst0 + (unsigned)(NOP * j + k) * 1024u);
        }
        piece((unsigned)(nblk * NOP + min(wave, scan_mats(KIND) - 1)) * 1024u, dst0 + 1024u * (NOP * NB));
        piece((unsigned)(nblk * NOP + scan_mats(KIND)) * 1024u, dst0 + 1024u * (NOP * NB + 1));  // w of all channels (and what lies behind it)
        const unsigned long long vbase = scalar(vp + (size_t)(DC * c) * a.ld * sizeof(T));
#pragma unroll
        for (int k = 0; k < L::VI; ++k) {
            const int t = min((64 / L::DW) * k + lane / L::DW, run.n_rows - 1 - DC * c);
            const unsigned off = (unsigned)(t * a.ld) * (unsigned)sizeof(T) + (unsigned)(lane % L::DW) * 4u;
            unsigned keep;
            asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %3\n\ts_nop 0\n\tglobal_load_lds_dword %1, %2\n\ts_mov_b32 m0, %0"
                         : "=&s"(keep)
                         : "v"(off), "s"(vbase), "s"(dst0 + 1024u * L::PIECES + 256u * k)
                         : "memory");
        }
    };
    const dr_f32x4 zero = {0.0f, 0.0f, 0.0f, 0.0f};
    auto store_o = [&](int c) {  // chunk c's outputs: one per thread
        const float *p = (const float *)s_o[c % L::PB] + threadIdx.x;
        const float o = (p[0] + p[256]) + (p[512] + p[768]);
        const int l = threadIdx.x >> 2, t = DC * c + 4 * (l >> 4) + (threadIdx.x & 3), d = 16 * cb + (l & 15);
        if (t < run.n_rows && d < V) a.o[((size_t)(run.row0 + t) * a.H + head) * a.V8 + d] = o;
    };
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // (the state's loads: the waits below count DMAs)
#pragma unroll
    for (int i = 0; i < L::RING - 1; ++i) fetch(c_lo + i, i);
    int at = 0;
    for (int c = c_lo; c < c_hi; ++c) {
        asm volatile("s_waitcnt vmcnt(%0)" ::"n"((L::RING - 2) * L::OPS) : "memory");
        fetch(c + L::RING - 1, at ? at - 1 : L::RING - 1);  // into the previous chunk's slot
        const char *mine = s_ring + at * L::SLOT + wave * L::WAVE;
        at = at + 1 < L::RING ? at + 1 : 0;
        auto operand = [&](int piece) { return *(const dr_f32x4 *)(mine + piece * 1024 + lane * 16); };
        dr_f32x4 u[NB], r[NB], k[NB], m[NB], w[NB], v, x = operand(NOP * NB);
        if constexpr (KIND != SCAN_LINEAR)
#pragma unroll
            for (int j = 0; j < NB; ++j) u[j] = operand(NOP * j);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = 4 * q + i;
            const float e = E::load((const T *)(mine + L::PIECES * 1024) + t * 16 + n16) + vbias;
            v[i] = DC * c + t < run.n_rows && col < V ? e : 0.0f;
        }
#pragma unroll
        for (int j = 0; j < NB; ++j) r[j] = operand(NOP * j + OR), k[j] = operand(NOP * j + OK), w[j] = *(const dr_f32x4 *)(mine + (NOP * NB + 1) * 1024 + (16 * min(wave * NB + j, nblk - 1) + 4 * q) * 4);
        dr_f32x4 P = zero, O = zero;
        if constexpr (KIND != SCAN_LINEAR) {
#pragma unroll
            for (int j = 0; j < NB; ++j)
#pragma unroll
                for (int i = 0; i < 4; ++i) P = dr_mfma(u[j][i], S[j][i], P);
            if (wave == 0)
#pragma unroll
                for (int i = 0; i < 4; ++i) P = dr_mfma(x[i], v[i], P);
            s_p[c % L::PB][wave][lane] = P;
        }
        if constexpr (KIND == SCAN_DELTA)
#pragma unroll
            for (int j = 0; j < NB; ++j) m[j] = operand(4 * j + 3);
#pragma unroll
        for (int j = 0; j < NB; ++j)
#pragma unroll
            for (int i = 0; i < 4; ++i) O = dr_mfma(r[j][i], S[j][i], O);
        if (KIND == SCAN_DELTA ? wave == 1 : KIND == SCAN_LINEAR && wave == 0)
#pragma unroll
            for (int i = 0; i < 4; ++i) O = dr_mfma(x[i], v[i], O);
#pragma unroll
        for (int j = 0; j < NB; ++j) S[j] *= w[j];
        if constexpr (KIND != SCAN_GATED)
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < NB; ++j) S[j] = dr_mfma(k[j][i], v[i], S[j]);
        // the four waves' shares of P (and of the previous outputs) meet (LDS only: the DMAs stay in flight)
        lds_barrier();
        if constexpr (KIND != SCAN_LINEAR) P = (s_p[c % L::PB][0][lane] + s_p[c % L::PB][1][lane]) + (s_p[c % L::PB][2][lane] + s_p[c % L::PB][3][lane]);
        if (c > c_lo) store_o(c - 1);
        if constexpr (KIND != SCAN_LINEAR) {
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < NB; ++j) S[j] = dr_mfma(KIND == SCAN_GATED ? k[j][i] : m[j][i], P[i], S[j]);
            if (wave == (KIND == SCAN_GATED ? 1 : 2))
#pragma unroll
                for (int i = 0; i < 4; ++i) O = dr_mfma(x[i], P[i], O);
        }
#pragma unroll
        for (int j = 0; j < NB; ++j)
            if (wave * NB + j >= nblk) S[j] = zero;  // (a block that does not exist saw another's operands)
        if constexpr (L::PB == 1) lds_barrier();  // everyone has read P and the previous outputs
        s_o[c % L::PB][wave][lane] = O;
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // the look-ahead DMAs: LDS is handed on when the workgroup ends
    __syncthreads();
    store_o(c_hi - 1);
#pragma unroll
    for (int j = 0; j < NB; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int d = 16 * (wave * NB + j) + 4 * q + i;
            if (d < D && col < V) state[(size_t)d * V + col] = S[j][i];
        }
}

// chunks whose operands are made and used at a time
int scan_segment(int kind, int H, int D) {
    const size_t bytes = H * scan_chunk_floats(kind, D) * 4;
    return (int)std::max((size_t)16, SCAN_SEGMENT_BYTES / bytes);
}
size_t scan_ws_floats(int kind, int chunks, int H, int D) { return (size_t)std::min(chunks, scan_segment(kind, H, D)) * H * scan_chunk_floats(kind, D); }
int scan_launches(int kind, int chunks, int H, int D) { return 2 * ((chunks + scan_segment(kind, H, D) - 1) / scan_segment(kind, H, D)); }

// prep(lo, hi): enqueues the preparation of chunks [lo, hi); a segment's operands are read back before they leave the last-level cache
template <class E, int NB, int KIND, class F>
int scan_chunks(ScanArgs a, int chunks, hipStream_t st, F &&prep) {
    const int step = scan_segment(KIND, a.H, a.D);
    for (int c = 0; c < chunks; c += step) {
        a.chunk_lo = c, a.chunk_hi = std::min(chunks, c + step);
        prep(a.chunk_lo, a.chunk_hi);
        PIE_LAUNCH_CHECK();
        hipLaunchKernelGGL((k_scan<E, NB, KIND>), dim3((unsigned)(a.H * dr_blocks(a.V)), (unsigned)a.n_runs), dim3(256), 0, st, a);
        PIE_LAUNCH_CHECK();
    }
    return PIE_OK;
}

}  // namespace
