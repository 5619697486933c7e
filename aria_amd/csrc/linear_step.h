// The linear-attention recurrence token by token (fp32 or bf16): the decode step, and the any-size form of a prompt.
#pragma once
#include "elem.h"

namespace ad {

__device__ __forceinline__ float silu_exact(float z) { return z * sigmoid_exact(z); }
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
    return (fminf(z, 0.f) - log1pf(expf(-fabsf(z)))) * s.inv_tau * 1.4426950408889634f;
}

struct StepOut {   // sums != NULL (one token a sequence): out = o w sigmoid(gate), and the sums of squares of o, [T, H, 16-column blocks]
    float* sums = nullptr;
    const float* w = nullptr;   // [H dvp]
    long long g_off = 0;        // gate columns of a proj row
};

namespace {
// grid (16-column blocks of the values, heads, sequences), 256 threads: thread (rl, cg) holds rows rl + 64 i of four state columns.  One token is the
// decode step; more are the any-size form of a prompt.
template <class T, int NR>
__global__ __launch_bounds__(256) void linear_step_kernel(const T* proj, AriaLinearShape s, float* state, const int32_t* slot, const int32_t* pos, const int32_t* cu,
                                                          T* out, StepOut so) {
    ARIA_SMEM_STATIC float sq[64 * NR], sk[64 * NR], sa[64 * NR], sv[16], red[4][16];
    const int t = threadIdx.x, l = t & 63, w = t >> 6, cg = t & 3, rl = t >> 2;
    const int v0 = blockIdx.x * 16, h = blockIdx.y, r0 = cu[blockIdx.z], r1 = cu[blockIdx.z + 1], dp = int(s.dp);
    if (r0 >= r1) return;
    const bool mine = v0 + 4 * cg < s.dvp;
    float* st = state + (((long long)slot[r0] * s.H + h) * dp) * s.dvp + v0 + 4 * cg;
    f32x4 S[NR];
#pragma unroll
    for (int i = 0; i < NR; ++i) S[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (pos[r0] > 0 && mine) {
#pragma unroll
        for (int i = 0; i < NR; ++i)
            if (rl + 64 * i < dp) S[i] = *reinterpret_cast<const f32x4*>(st + (long long)(rl + 64 * i) * s.dvp);
    }
    for (int row = r0; row < r1; ++row) {
        const T* p = proj + (long long)row * s.ldp;
        for (int d = t; d < 64 * NR; d += 256) {
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
        if (t < 16) {
            float v = v0 + t < s.dvp ? ldf(p + s.v_off + h * s.dvp + v0 + t) : 0.f;
            sv[t] = s.silu ? silu_exact(v) : v;
        }
        sync();
        f32x4 o = f32x4{0.f, 0.f, 0.f, 0.f};
        const f32x4 v = *reinterpret_cast<const f32x4*>(sv + 4 * cg);
#pragma unroll
        for (int i = 0; i < NR; ++i) {
            const float q = sq[rl + 64 * i], k = sk[rl + 64 * i], a = sa[rl + 64 * i];
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                S[i][e] = a * S[i][e] + k * v[e];
                o[e] += S[i][e] * q;
            }
        }
#pragma unroll
        for (int e = 0; e < 4; ++e)
#pragma unroll
            for (int m = 4; m < 64; m <<= 1) o[e] += shfl_xor(o[e], m);
        if (l < 4) {
#pragma unroll
            for (int e = 0; e < 4; ++e) red[w][4 * l + e] = o[e];
        }
        sync();
        if (w == 0) {   // (every 16 lanes the same outputs)
            const int c = l & 15, col = h * int(s.dvp) + v0 + c;
            const bool in = v0 + c < s.dvp;
            float y = in ? (red[0][c] + red[1][c]) + (red[2][c] + red[3][c]) : 0.f;
            if (so.sums) {   // (one token) the squares of the outputs, which leave with their norm's weight and their gate but without 1 / rms
                const float ss = group_sum<16>(y * y);
                if (l == 0) so.sums[((long long)row * gridDim.y + h) * gridDim.x + blockIdx.x] = ss;
                if (in) y *= so.w[col] * sigmoid_exact(ldf(p + so.g_off + col));
            }
            if (in && l < 16) stf(out + (long long)row * s.H * s.dvp + col, y);
        }
    }
    if (mine) {
#pragma unroll
        for (int i = 0; i < NR; ++i)
            if (rl + 64 * i < dp) *reinterpret_cast<f32x4*>(st + (long long)(rl + 64 * i) * s.dvp) = S[i];
    }
}

template <class T>
int launch_step(const void* proj, const AriaLinearShape& s, float* state, const int32_t* slot, const int32_t* pos, const int32_t* cu, int64_t n_seq, void* out,
                const StepOut& so, void* stream) {
    const dim3 grid(unsigned((s.dvp + 15) / 16), unsigned(s.H), unsigned(n_seq)), block(256);
#define ARIA_STEP(N) ARIA_LAUNCH((linear_step_kernel<T, N>), grid, block, 0, stream, static_cast<const T*>(proj), s, state, slot, pos, cu, static_cast<T*>(out), so)
    if (s.dp <= 64)
        ARIA_STEP(1);
    else if (s.dp <= 128)
        ARIA_STEP(2);
    else if (s.dp <= 256)
        ARIA_STEP(4);
    else if (s.dp <= 512)
        ARIA_STEP(8);
    else
        ARIA_STEP(16);
#undef ARIA_STEP
    return aria_check_launch();
}
}  // namespace
}  // namespace ad
