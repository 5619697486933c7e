// Element access shared by the kernels that exist in a bfloat16 and a 32-bit form, the dynamic-tanh norm, and the two routing / activation
// formulas those kernels share.
#pragma once
#include "aria_device.h"
#include "aria_hip.h"
#include <cmath>

namespace ad {

__device__ __forceinline__ float ldf(const bf16_t* p) { return bf2f(*p); }
__device__ __forceinline__ float ldf(const float* p) { return *p; }
__device__ __forceinline__ void stf(bf16_t* p, float v) { *p = f2bf(v); }
__device__ __forceinline__ void stf(float* p, float v) { *p = v; }
// 8 consecutive elements (16-byte aligned)
__device__ __forceinline__ void ld8(const bf16_t* p, float (&v)[8]) {
    const u32x4 a = ld16(p);
#pragma unroll
    for (int q = 0; q < 4; ++q) {
        v[2 * q] = bflo(a[q]);
        v[2 * q + 1] = bfhi(a[q]);
    }
}
__device__ __forceinline__ void ld8(const float* p, float (&v)[8]) {
    const f32x4 a = *reinterpret_cast<const f32x4*>(p), b = *reinterpret_cast<const f32x4*>(p + 4);
#pragma unroll
    for (int q = 0; q < 4; ++q) {
        v[q] = a[q];
        v[4 + q] = b[q];
    }
}
__device__ __forceinline__ void st8(bf16_t* p, const float (&v)[8]) {
    st16(p, u32x4{pack2bf(v[0], v[1]), pack2bf(v[2], v[3]), pack2bf(v[4], v[5]), pack2bf(v[6], v[7])});
}
__device__ __forceinline__ void st8(float* p, const float (&v)[8]) {
    *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
    *reinterpret_cast<f32x4*>(p + 4) = f32x4{v[4], v[5], v[6], v[7]};
}

// wave_max_bcast of N values, their DPP ladders in step (one ladder alone is a chain of dependent instructions)
template <int N>
__device__ __forceinline__ void wave_max_bcast_n(float (&v)[N]) {
#ifdef ARIA_EMU
    for (int j = 0; j < N; ++j) v[j] = wave_max_bcast(v[j]);
#else
    const int ninf = int(0xff800000u);
#define ARIA_DPP_MAXN(ctrl, rows)        \
    _Pragma("unroll") for (int j = 0; j < N; ++j) v[j] = \
        fmaxf(v[j], __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(ninf, __builtin_bit_cast(int, v[j]), ctrl, rows, 0xF, false)))
    ARIA_DPP_MAXN(0x111, 0xF);  // row_shr:1, 2, 4, 8: lane 15 of every row holds the row's maximum
    ARIA_DPP_MAXN(0x112, 0xF);
    ARIA_DPP_MAXN(0x114, 0xF);
    ARIA_DPP_MAXN(0x118, 0xF);
    ARIA_DPP_MAXN(0x142, 0xA);  // row_bcast:15, 31
    ARIA_DPP_MAXN(0x143, 0xC);
#undef ARIA_DPP_MAXN
#pragma unroll
    for (int j = 0; j < N; ++j) v[j] = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v[j]), 63));
#endif
}

// tanh: the 32-bit form is libm's; beside bfloat16 activations 1 - 2 / (1 + e^2z) on v_exp_f32 + v_rcp_f32 (absolute error ~1e-7)
template <class T>
__device__ __forceinline__ float tanh_for(float z);
template <>
__device__ __forceinline__ float tanh_for<float>(float z) { return tanhf(z); }
template <>
__device__ __forceinline__ float tanh_for<bf16_t>(float z) { return 1.f - 2.f * rcp_fast(1.f + exp2_fast(2.8853900817779268f * z)); }

// Dynamic tanh ("norm" without statistics): tanh(alpha v) w[n] + b[n]
template <class T>
__device__ __forceinline__ float dyt(const AriaDyT& p, float v, int n) { return tanh_for<T>(p.alpha * v) * p.w[n] + p.b[n]; }

__device__ __forceinline__ float sigmoid_exact(float z) { return 1.f / (1.f + expf(-z)); }
__device__ __forceinline__ float softcap(float z, float cap) { return cap * tanhf(z / cap); }
__device__ __forceinline__ float relu_squared(float z) {
    const float r = fmaxf(z, 0.f);
    return r * r;
}

// Group-limited routing of ONE token by one wave.  s = sigmoid(logit); choice = s + correction; experts form `groups` equal groups of
// neighbours, a group ranks by the sum of its two largest choice scores, the best `keep` groups stay, and of their experts the k with the
// largest choice scores are taken (ties to the lower id).  Lane j < k returns expert j and its weight s; `want`: the expert of that slot as a
// wave-uniform value.  lds: 3 * 256 floats of this wave.  E <= 256, k <= 64.
__device__ __forceinline__ int route_group_limited(const float* logits, const float* correction, int E, int groups, int keep, int k, float* lds,
                                                   int l, int want, float& my_w, int& my_e) {
    float *choice = lds, *sig = lds + 256, *gsum = lds + 512;
    float v[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int e = l + 64 * i;
        v[i] = -INFINITY;
        if (e < E) {
            const float s = sigmoid_exact(logits[e]);
            v[i] = s + correction[e];
            choice[e] = v[i];
            sig[e] = s;
        }
    }
    wave_barrier();
    const int size = E / groups;
    if (keep < groups) {   // (wave-uniform)
        for (int g = l; g < groups; g += 64) {
            float a = -INFINITY, b = -INFINITY;
            for (int i = 0; i < size; ++i) {
                const float c = choice[g * size + i];
                if (c > a) {
                    b = a;
                    a = c;
                } else if (c > b) {
                    b = c;
                }
            }
            gsum[g] = size > 1 ? a + b : a;
        }
        wave_barrier();
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int e = l + 64 * i;
            if (e < E) {
                const int g = e / size;
                const float mine = gsum[g];
                int better = 0;
                for (int o = 0; o < groups; ++o) better += gsum[o] > mine || (gsum[o] == mine && o < g);
                if (better >= keep) v[i] = -INFINITY;
            }
        }
    }
    int wanted = 0;
    my_e = 0;
    for (int j = 0; j < k; ++j) {
        const float m = wave_max_bcast(fmaxf(fmaxf(v[0], v[1]), fmaxf(v[2], v[3])));
        int bi = -1;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const unsigned long long hit = ballot(v[i] == m && l + 64 * i < E);
            if (bi < 0 && hit) bi = __builtin_ctzll(hit) + 64 * i;
        }
        if (bi < 0) bi = 0;  // (NaN scores: stay in range)
        if (l == j) my_e = bi;
        if (j == want) wanted = bi;
        if ((bi & 63) == l) {
#pragma unroll
            for (int i = 0; i < 4; ++i)
                if (i == (bi >> 6)) v[i] = -INFINITY;
        }
    }
    my_w = sig[my_e];
    wave_barrier();
    return wanted;
}

}  // namespace ad
