// delta_rule.hip -- the generalised delta rule (PIE_MIXER_DELTA): per head a state S [key channel][value column] in fp32, carried from token to token,
//   S_t = diag(w_t) S_(t-1) - (a_t u_t) (u_t^T S_(t-1)) + k_t v_t^T,   o_t = S_t^T r_t,
// with the unit key u = k / sqrt(sum k^2 + unit_eps), the decay w = exp(-decay_scale sigmoid(.)) and the removal rate a = sigmoid(.), all fp32.
//
// Step form (decoded tokens, short runs): one workgroup per (run, head).  A thread keeps RPT key channels of one value column in registers; the channel
// vectors of a token are broadcast from LDS.  Columns are independent, so a token costs two exchanges between the channel slices: u^T S and r^T S.
// The decay's low-rank projection, the unit key, the head's norm and the output gate are taken on the way.
#include "stack_types.hpp"

namespace {


template <class E, int CP, int NT>  // CP: power of two >= D; NT threads
__global__ void __launch_bounds__(NT) k_delta_step(const DeltaArgs a) {
    typedef typename E::type T;
    constexpr int SL = NT / CP, RPT = CP / SL;  // channel slices; channels per thread
    static_assert(NT % CP == 0 && CP % SL == 0 && NT % 64 == 0, "slices");
    __shared__ __attribute__((aligned(16))) float s_r[CP], s_k[CP], s_v[CP], s_g[CP], s_a[CP], s_w[CP], s_low[DELTA_MAX_RANK], s_p[SL][CP], s_o[SL][CP], s_ss[NT / 64];
    const int run_i = blockIdx.x, head = blockIdx.y, D = a.D, lane = threadIdx.x & 63;
    const RowRun run = a.runs[run_i];
    const int col = threadIdx.x % CP, slice = threadIdx.x / CP, d0 = slice * RPT;
    const int seq = min(a.row_seq[run.row0], a.n_seqs - 1);
    const size_t slot = min((unsigned)a.slots[seq], (unsigned)a.n_slots - 1u);
    float *state = a.state + (slot * a.H + head) * D * D;
    float S[RPT];
    const bool fresh = a.pos[run.row0] == 0;
#pragma unroll
    for (int i = 0; i < RPT; ++i) S[i] = !fresh && col < D && d0 + i < D ? state[(size_t)(d0 + i) * D + col] : 0.0f;
    const int HD8 = a.H * a.D8;

    for (int j = 0; j < run.n_rows; ++j) {
        const size_t m = run.row0 + j;
        const T *x = (const T *)a.raw + m * a.ld + head * a.D8;
        const u16 *bias = a.bias ? a.bias + head * a.D8 : nullptr;
        for (int i = threadIdx.x; i < 5 * CP; i += NT) {  // r, k, v, gate, rate; channels past D: nothing
            const int what = i / CP, d = i % CP;
            float v = d < D ? E::load(x + what * HD8 + d) + (bias ? BF16::to_f32(bias[what * HD8 + d]) : 0.0f) : 0.0f;
            if (what >= 3) v = d < D ? 1.0f / (1.0f + expf(-v)) : 0.0f;
            float *dst = what == 0 ? s_r : what == 1 ? s_k : what == 2 ? s_v : what == 3 ? s_g : s_a;
            dst[d] = v;
        }
        for (int i = threadIdx.x; i < a.R8; i += NT) {
            const float z = i < a.rank ? E::load((const T *)a.raw + m * a.ld + 5 * HD8 + i) + (a.bias ? BF16::to_f32(a.bias[5 * HD8 + i]) : 0.0f) : 0.0f;
            s_low[i] = tanhf(z);
        }
        __syncthreads();
        // the decay: eight lanes per channel
        for (int d = threadIdx.x >> 3; d < CP; d += NT / 8) {
            float z = 0.0f;
            if (d < D) {
                const u16 *wr = a.w_decay + (size_t)(head * D + d) * a.R8;
                for (int i = (threadIdx.x & 7) * 8; i < a.R8; i += 64) {
                    const uint4 q = *(const uint4 *)(wr + i);
                    const float4 l0 = *(const float4 *)(s_low + i), l1 = *(const float4 *)(s_low + i + 4);
                    z = fmaf(lo_f32<BF16>(q.x), l0.x, fmaf(hi_f32<BF16>(q.x), l0.y, fmaf(lo_f32<BF16>(q.y), l0.z, fmaf(hi_f32<BF16>(q.y), l0.w, z))));
                    z = fmaf(lo_f32<BF16>(q.z), l1.x, fmaf(hi_f32<BF16>(q.z), l1.y, fmaf(lo_f32<BF16>(q.w), l1.z, fmaf(hi_f32<BF16>(q.w), l1.w, z))));
                }
            }
            z = lanes8_sum(z);
            if ((threadIdx.x & 7) == 0) s_w[d] = d < D ? expf(-a.decay_scale / (1.0f + expf(-(z + a.decay_bias[head * D + d])))) : 1.0f;
        }
        float ss = 0.0f;  // every wave: the key's length
        for (int d = lane; d < CP; d += 64) ss = fmaf(s_k[d], s_k[d], ss);
        const float unit = 1.0f / sqrtf(wave_sum(ss) + a.unit_eps);
        float p = 0.0f;
#pragma unroll
        for (int i = 0; i < RPT; ++i) p = fmaf(s_k[d0 + i], S[i], p);
        s_p[slice][col] = p * unit;
        __syncthreads();
        p = 0.0f;
#pragma unroll
        for (int i = 0; i < SL; ++i) p += s_p[i][col];
        const float v = s_v[col];
        float o = 0.0f;
#pragma unroll
        for (int i = 0; i < RPT; ++i) {
            const float k = s_k[d0 + i];
            S[i] = fmaf(k, v, fmaf(-(s_a[d0 + i] * k * unit), p, s_w[d0 + i] * S[i]));
            o = fmaf(s_r[d0 + i], S[i], o);
        }
        s_o[slice][col] = o;
        __syncthreads();
        if (threadIdx.x < (CP < 64 ? 64 : CP)) {  // whole waves
            o = 0.0f;
            if (threadIdx.x < CP)
#pragma unroll
                for (int i = 0; i < SL; ++i) o += s_o[i][col];
            const float sum = wave_sum(o * o);
            if (lane == 0) s_ss[threadIdx.x >> 6] = sum;
        }
        __syncthreads();
        if (threadIdx.x < D) {
            float sum = s_ss[0];
#pragma unroll
            for (int i = 1; i < (CP + 63) / 64; ++i) sum += s_ss[i];
            const float y = o * (1.0f / sqrtf(sum / (float)D + a.eps)) * a.o_norm[head * D + threadIdx.x] * s_g[threadIdx.x];
            ((T *)a.out)[m * a.ld_out + head * a.D8 + threadIdx.x] = E::pack(y);
        }
        __syncthreads();  // the channel vectors are written again
    }
    if (col < D)
#pragma unroll
        for (int i = 0; i < RPT; ++i)
            if (d0 + i < D) state[(size_t)(d0 + i) * D + col] = S[i];
}

template <class E>
int delta_step_go(const DeltaArgs &a, hipStream_t st) {
    const dim3 grid((unsigned)a.n_runs, (unsigned)a.H);
#define DS_GO(CP_, NT_) hipLaunchKernelGGL((k_delta_step<E, CP_, NT_>), grid, dim3(NT_), 0, st, a)
    if (a.D <= 16) DS_GO(16, 128);
    else if (a.D <= 32) DS_GO(32, 256);
    else if (a.D <= 64) DS_GO(64, 256);
    else if (a.D <= 128) DS_GO(128, 512);
    else DS_GO(256, 1024);
#undef DS_GO
    PIE_LAUNCH_CHECK();
    return PIE_OK;
}

}  // namespace

int delta_step_launch(int dtype, const DeltaArgs &a, hipStream_t st) {
    if (a.n_runs <= 0) return PIE_OK;
    PIE_REQUIRE(a.D > 0 && a.D <= DELTA_MAX_DIM && a.rank > 0 && a.rank <= DELTA_MAX_RANK && a.H > 0 && a.H <= 65535, PIE_E_SHAPE,
                "delta rule: heads of at most 256 channels, decay rank of at most 1024");
    PIE_REQUIRE(a.slots && a.state && a.n_slots > 0, PIE_E_ARG, "delta rule: no state slots");
    return dtype == PIE_F32 ? delta_step_go<ElemF32>(a, st) : delta_step_go<ElemBF16>(a, st);
}
