// The linear-attention recurrence token by token (fp32 or bf16): the decode step, and the any-size form of a prompt.
#pragma once
#include "elem.h"

namespace ad {

__device__ __forceinline__ float silu_exact(float z) { return z * sigmoid_exact(z); }
// log2 of sigmoid(z) without cancellation: min(z, 0) - log(1 + e^-|z|)
__device__ __forceinline__ float log2_sigmoid(float z) {
    return fminf(z, 0.f) * 1.4426950408889634f - log2f(1.f + exp2f(-1.4426950408889634f * fabsf(z)));
}
// the same on v_exp_f32 and v_log_f32 (1 ulp each)
__device__ __forceinline__ float log2_sigmoid_fast(float z) {
    const float t = 1.4426950408889634f * z;
    return fminf(t, 0.f) - log2_fast(1.f + exp2_fast(-fabsf(t)));
}
// log2 of the gated decay of channel i (over all heads): sigmoid(a2 a1 + b)^inv_tau, the logarithm of the sigmoid without cancellation
template <class T>
__device__ __forceinline__ float gate_log2(const AriaLinearShape& s, const T* a1, int i) {
    const T* w = static_cast<const T*>(s.a2) + (long long)i * s.rank;
    float z = s.a_bias[i];
    for (int r = 0; r < s.rank; r += 8) {
        float a[8], b[8];
        ld8(w + r, a);
        ld8(a1 + r, b);
#pragma unroll
        for (int e = 0; e < 8; ++e) z += a[e] * b[e];
    }
    return log2_sigmoid(z) * s.inv_tau;
}

struct StepOut {   // sums != NULL (one token a sequence): out = o w sigmoid(gate), and the sums of squares of o, [T, H, blocks]
    float* sums = nullptr;
    const float* w = nullptr;   // [H dvp]
    long long g_off = 0;        // gate columns of a proj row
};

namespace {
// grid (4 CG-column blocks of the values, heads, sequences), 256 threads: thread (rl, cg) holds rows rl + RL i of four state columns.  One token is the
// decode step; more are the any-size form of a prompt.  CG = 8: whole 128-byte lines of the state; CG = 4: more workgroups where there are few.
template <class T, int NR, int CG>
__global__ __launch_bounds__(256) void linear_step_kernel(const T* proj, AriaLinearShape s, float* state, const int32_t* slot, const int32_t* pos, const int32_t* cu,
                                                          T* out, StepOut so) {
    constexpr int RL = 256 / CG, VB = 4 * CG, ROWS = RL * NR;
    ARIA_SMEM_STATIC float sq[ROWS], sk[ROWS], sa[ROWS], sv[VB], red[4][VB];
    const int t = threadIdx.x, l = t & 63, w = t >> 6, cg = t % CG, rl = t / CG;
    const int v0 = blockIdx.x * VB, h = blockIdx.y, dp = int(s.dp);
    const int r0 = cu ? cu[blockIdx.z] : int(blockIdx.z), r1 = cu ? cu[blockIdx.z + 1] : r0 + 1;   // (no cu: one token a sequence)
    if (r0 >= r1) return;
    const bool mine = v0 + 4 * cg < s.dvp;
    float* st = state + (((long long)slot[r0] * s.H + h) * dp) * s.dvp + v0 + 4 * cg;
    f32x4 S[NR];
#pragma unroll
    for (int i = 0; i < NR; ++i) S[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (pos[r0] > 0 && mine) {
#pragma unroll
        for (int i = 0; i < NR; ++i)
            if (rl + RL * i < dp) S[i] = *reinterpret_cast<const f32x4*>(st + (long long)(rl + RL * i) * s.dvp);
    }
    for (int row = r0; row < r1; ++row) {
        const T* p = proj + (long long)row * s.ldp;
        for (int d = t; d < ROWS; d += 256) {
            float q = 0.f, k = 0.f, a = 1.f;
            if (d < dp) {
                q = ldf(p + s.q_off + h * dp + d);
                k = ldf(p + s.k_off + h * dp + d);
                a = s.decay ? s.decay[2 * h] : exp2f(gate_log2(s, p + s.a_off, h * dp + d));
                if (s.silu) q = silu_exact(q), k = silu_exact(k);
            }
            sq[d] = q * s.q_scale;
            sk[d] = k;
            sa[d] = a;
        }
        if (t < VB) {
            float v = v0 + t < s.dvp ? ldf(p + s.v_off + h * s.dvp + v0 + t) : 0.f;
            sv[t] = s.silu ? silu_exact(v) : v;
        }
        sync();
        f32x4 o = f32x4{0.f, 0.f, 0.f, 0.f};
        const f32x4 v = *reinterpret_cast<const f32x4*>(sv + 4 * cg);
#pragma unroll
        for (int i = 0; i < NR; ++i) {
            const float q = sq[rl + RL * i], k = sk[rl + RL * i], a = sa[rl + RL * i];
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                S[i][e] = a * S[i][e] + k * v[e];
                o[e] += S[i][e] * q;
            }
        }
#pragma unroll
        for (int e = 0; e < 4; ++e)
#pragma unroll
            for (int m = CG; m < 64; m <<= 1) o[e] += shfl_xor(o[e], m);
        if (l < CG) {
#pragma unroll
            for (int e = 0; e < 4; ++e) red[w][4 * l + e] = o[e];
        }
        sync();
        if (w == 0) {   // (lanes past the block repeat it)
            const int c = l % VB, col = h * int(s.dvp) + v0 + c;
            const bool in = v0 + c < s.dvp;
            float y = in ? (red[0][c] + red[1][c]) + (red[2][c] + red[3][c]) : 0.f;
            if (so.sums) {   // (one token) the squares of the outputs, which leave with their norm's weight and their gate but without 1 / rms
                float ss = group_sum<16>(y * y);
                if (VB == 32) ss += shfl_xor(ss, 16);
                if (l == 0) so.sums[((long long)row * gridDim.y + h) * gridDim.x + blockIdx.x] = ss;
                if (in) y *= so.w[col] * sigmoid_exact(ldf(p + so.g_off + col));
            }
            if (in && l < VB) stf(out + (long long)row * s.H * s.dvp + col, y);
        }
    }
    if (mine) {
#pragma unroll
        for (int i = 0; i < NR; ++i)
            if (rl + RL * i < dp) *reinterpret_cast<f32x4*>(st + (long long)(rl + RL * i) * s.dvp) = S[i];
    }
}

// value columns of a workgroup
inline int step_columns(const AriaLinearShape& s, int64_t n_seq) { return s.dp <= 512 && n_seq * s.H * ((s.dvp + 31) / 32) >= 512 ? 32 : 16; }
inline int64_t step_blocks(const AriaLinearShape& s, int64_t n_seq) { return (s.dvp + step_columns(s, n_seq) - 1) / step_columns(s, n_seq); }
template <class T>
int launch_step(const void* proj, const AriaLinearShape& s, float* state, const int32_t* slot, const int32_t* pos, const int32_t* cu, int64_t n_seq, void* out,
                const StepOut& so, void* stream) {
    const dim3 grid(unsigned(step_blocks(s, n_seq)), unsigned(s.H), unsigned(n_seq)), block(256);
#define ARIA_STEP(N, C) \
    ARIA_LAUNCH((linear_step_kernel<T, N, C>), grid, block, 0, stream, static_cast<const T*>(proj), s, state, slot, pos, cu, static_cast<T*>(out), so)
    if (step_columns(s, n_seq) == 32) {
        if (s.dp <= 64)
            ARIA_STEP(2, 8);
        else if (s.dp <= 128)
            ARIA_STEP(4, 8);
        else if (s.dp <= 256)
            ARIA_STEP(8, 8);
        else
            ARIA_STEP(16, 8);
    } else {
        if (s.dp <= 64)
            ARIA_STEP(1, 4);
        else if (s.dp <= 128)
            ARIA_STEP(2, 4);
        else if (s.dp <= 256)
            ARIA_STEP(4, 4);
        else if (s.dp <= 512)
            ARIA_STEP(8, 4);
        else
            ARIA_STEP(16, 4);
    }
#undef ARIA_STEP
    return aria_check_launch();
}
}  // namespace
}  // namespace ad
