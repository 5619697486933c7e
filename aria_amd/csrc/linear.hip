// Linear attention: per head a matrix state S [d, dv] that decays, S_t = diag(a_t) S_(t-1) + k_t v_t^T, and is read by the query, o_t = S_t^T q_t.  The
// decay is one constant per head, or comes per token and key channel from a low-rank projection, a = sigmoid(a2 a1 + b)^(1 / tau).  States are fp32
// and live in the sequence's cache slot; a sequence at position 0 starts from zeros whatever the slot holds.
#include "elem.h"

namespace {
using namespace ad;
typedef AriaLinearShape Lin;

bool al16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

__device__ __forceinline__ float silu_exact(float z) { return z * sigmoid_exact(z); }
// log2 of the gated decay of channel i (over all heads): sigmoid(a2 a1 + b)^inv_tau, the logarithm of the sigmoid without cancellation
template <class T>
__device__ __forceinline__ float gate_log2(const Lin& s, const T* a1, int i) {
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

// ---------------------------------------------------------------------------------------------- token by token (fp32 or bf16)
// grid (16-column blocks of the values, heads, sequences), 256 threads: thread (rl, cg) holds rows rl + 64 i of four state columns.  One token is the
// decode step; more are the any-size form of a prompt.
template <class T, int NR>
__global__ __launch_bounds__(256) void linear_step_kernel(const T* proj, Lin s, float* state, const int32_t* slot, const int32_t* pos, const int32_t* cu, T* out) {
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
        if (t < 16 && v0 + t < s.dvp)
            stf(out + ((long long)row * s.H + h) * s.dvp + v0 + t, (red[0][t] + red[1][t]) + (red[2][t] + red[3][t]));
    }
    if (mine) {
#pragma unroll
        for (int i = 0; i < NR; ++i)
            if (rl + 64 * i < dp) *reinterpret_cast<f32x4*>(st + (long long)(rl + 64 * i) * s.dvp) = S[i];
    }
}

// ---------------------------------------------------------------------------------------------- norm per group of columns, times a gate
// a wave per (row, group)
template <class T>
__global__ __launch_bounds__(256) void norm_gate_kernel(const T* o, const T* gate, long long ldg, const float* w, long long w_stride, T* y, long long n_items,
                                                        int groups, int cols, float inv_n, float eps, int silu) {
    const int l = threadIdx.x & 63, nch = cols >> 3;
    const long long item = (long long)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (item >= n_items) return;
    const long long t = item / groups;
    const int g = int(item % groups);
    const T* src = o + item * cols;
    const T* gr = gate + t * ldg + (long long)g * cols;
    const float* wr = w + g * w_stride;
    float ss = 0.f;
    for (int c = l; c < nch; c += 64) {
        float v[8];
        ld8(src + c * 8, v);
#pragma unroll
        for (int e = 0; e < 8; ++e) ss += v[e] * v[e];
    }
    const float r = 1.f / sqrtf(wave_sum_bcast(ss) * inv_n + eps);
    for (int c = l; c < nch; c += 64) {
        float v[8], gv[8], wv[8];
        ld8(src + c * 8, v);
        ld8(gr + c * 8, gv);
        ld8(wr + c * 8, wv);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = v[e] * r * wv[e] * (silu ? silu_exact(gv[e]) : sigmoid_exact(gv[e]));
        st8(y + item * cols + c * 8, v);
    }
}

int shape_ok(const Lin* s) {
    if (!s || s->H <= 0 || s->d <= 0 || s->dv <= 0 || s->dp < s->d || s->dvp < s->dv || s->rank < 0) return ARIA_ERR_INVALID;
    if (!s->decay && (!s->a2 || !s->a_bias || s->rank <= 0 || s->a_off + s->rank > s->ldp)) return ARIA_ERR_INVALID;
    if (s->q_off + s->H * s->dp > s->ldp || s->k_off + s->H * s->dp > s->ldp || s->v_off + s->H * s->dvp > s->ldp) return ARIA_ERR_INVALID;
    if ((s->dp & 7) || (s->dvp & 7) || (s->ldp & 7) || (s->q_off & 7) || (s->k_off & 7) || (s->v_off & 7) || (s->a_off & 7) || (s->rank & 7) ||
        (s->a2 && !al16(s->a2)))
        return ARIA_ERR_ALIGN;
    return ARIA_OK;
}

template <class T>
int launch_step(const void* proj, const Lin& s, float* state, const int32_t* slot, const int32_t* pos, const int32_t* cu, int64_t n_seq, void* out, void* stream) {
    const dim3 grid(unsigned((s.dvp + 15) / 16), unsigned(s.H), unsigned(n_seq)), block(256);
#define ARIA_STEP(N) ARIA_LAUNCH((linear_step_kernel<T, N>), grid, block, 0, stream, static_cast<const T*>(proj), s, state, slot, pos, cu, static_cast<T*>(out))
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

extern "C" {

int aria_linear_step(const void* proj, const AriaLinearShape* s, float* state, const int32_t* slot, const int32_t* pos, const int32_t* cu, int64_t n_seq,
                     void* out, int f32, void* stream) {
    if (!proj || !state || !slot || !pos || !cu || !out || n_seq < 0) return ARIA_ERR_INVALID;
    if (const int rc = shape_ok(s)) return rc;
    if (!al16(proj) || !al16(state)) return ARIA_ERR_ALIGN;
    if (s->dp > 1024 || s->H > 65535 || n_seq > 65535) return ARIA_ERR_UNSUPPORTED;
    if (n_seq == 0) return ARIA_OK;
    return f32 ? launch_step<float>(proj, *s, state, slot, pos, cu, n_seq, out, stream) : launch_step<bf16_t>(proj, *s, state, slot, pos, cu, n_seq, out, stream);
}

int aria_norm_gate(const void* o, const void* gate, int64_t ldg, const float* w, int64_t w_stride, void* y, int64_t T, int64_t groups, int64_t cols, int64_t n,
                   float eps, int silu, int f32, void* stream) {
    if (!o || !gate || !w || !y || T < 0 || groups <= 0 || cols <= 0 || n <= 0 || n > cols) return ARIA_ERR_INVALID;
    if ((cols & 7) || (ldg & 7) || (w_stride & 3) || !al16(o) || !al16(gate) || !al16(w) || !al16(y)) return ARIA_ERR_ALIGN;
    if (T == 0) return ARIA_OK;
    const long long items = T * groups;
    const dim3 grid(unsigned((items + 3) / 4)), block(256);
    if (f32)
        ARIA_LAUNCH((norm_gate_kernel<float>), grid, block, 0, stream, static_cast<const float*>(o), static_cast<const float*>(gate), (long long)ldg, w,
                    (long long)w_stride, static_cast<float*>(y), items, int(groups), int(cols), 1.f / float(n), eps, silu);
    else
        ARIA_LAUNCH((norm_gate_kernel<bf16_t>), grid, block, 0, stream, static_cast<const bf16_t*>(o), static_cast<const bf16_t*>(gate), (long long)ldg, w,
                    (long long)w_stride, static_cast<bf16_t*>(y), items, int(groups), int(cols), 1.f / float(n), eps, silu);
    return aria_check_launch();
}

}  // extern "C"
