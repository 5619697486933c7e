// Row-streaming projections of 1 .. 16 tokens (bf16): the decode steps' matrix products, each with its consumer's elementwise work as an epilogue.
//
// An epilogue E is called once per output, e(value, token, row, problem).  E::SUMSQ: it returns the square of what it stored and offers `sums`, which
// receives per token and workgroup the sum of those squares -- partial sums for an RMS norm whose 1 / rms the CONSUMER of the stored rows applies to its
// results (RowsIn::sq): W (r x) = r (W x), so no launch of its own stands between the two.
#pragma once
#include "elem.h"

namespace ad {

__device__ __forceinline__ u32x4 ldw16(const bf16_t* p) {   // a weight stream is read once: non-temporal
#ifdef ARIA_EMU
    return ld16(p);
#else
    return __builtin_nontemporal_load(reinterpret_cast<const u32x4*>(p));
#endif
}
// acc[r][b] += W[row r] . X[token b], a wave over two weight rows and NB token rows: four 16-byte chunks per row and lane requested before the
// first use, the token rows come from the L1 / L2
template <int NB>
__device__ __forceinline__ void two_rows(float (&acc)[2][NB], const bf16_t* w0, const bf16_t* w1, const bf16_t* x, long long ldx, int nb, int K, int l) {
    const int nch = K >> 3;
    for (int c0 = l; c0 < nch; c0 += 256) {
        u32x4 a[2][4];
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int c = min(c0 + 64 * u, nch - 1);
            a[0][u] = ldw16(w0 + c * 8);
            a[1][u] = ldw16(w1 + c * 8);
        }
#pragma unroll
        for (int b = 0; b < NB; ++b) {
            const bf16_t* xr = x + (long long)min(b, nb - 1) * ldx;
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                u32x4 v = ld16(xr + min(c0 + 64 * u, nch - 1) * 8);
                const bool in = c0 + 64 * u < nch;
#pragma unroll
                for (int q = 0; q < 4; ++q) {
                    const uint32_t xv = in ? v[q] : 0u;
                    acc[0][b] = dot2bf(a[0][u][q], xv, acc[0][b]);
                    acc[1][b] = dot2bf(a[1][u][q], xv, acc[1][b]);
                }
            }
        }
    }
#pragma unroll
    for (int r = 0; r < 2; ++r)
#pragma unroll
        for (int b = 0; b < NB; ++b) acc[r][b] = wave_sum_bcast(acc[r][b]);
}

struct RowsIn {
    const bf16_t* W;    // [N, K]
    const bf16_t* W2;   // second matrix of a gated pair
    const bf16_t* X;    // [T, ldx]
    long long ldx;
    int K, N;
    const float* sq = nullptr;   // [T, sq_n] partial sums of squares: results are multiplied by 1 / sqrt(sum inv_n + eps)
    int sq_n = 0;
    float inv_n = 0.f, eps = 0.f;
};
struct RowsPair {   // up to two problems of one launch (blockIdx.z): equal N and tokens
    RowsIn in[2];
};

namespace {
// one token: a wave per two weight rows (PAIR: per output, gate row and up row)
template <class E, bool PAIR>
__global__ __launch_bounds__(256) void row_kernel(RowsPair rp, E e) {
    ARIA_SMEM_STATIC float red[8];
    const RowsIn& in = rp.in[blockIdx.z];
    const int t = threadIdx.x, l = t & 63, w = t >> 6, N = in.N;
    const int row0 = PAIR ? blockIdx.x * 4 + w : (blockIdx.x * 4 + w) * 2;
    const int r0 = min(row0, N - 1), r1 = PAIR ? r0 : min(row0 + 1, N - 1);
    float ss = 0.f;
    if (in.sq) {
        for (int i = t; i < in.sq_n; i += 256) ss += in.sq[i];
    }
    float acc[2][1] = {{0.f}, {0.f}};
    two_rows<1>(acc, in.W + (long long)r0 * in.K, (PAIR ? in.W2 : in.W) + (long long)r1 * in.K, in.X, 0, 1, in.K, l);
    float v0 = acc[0][0], v1 = acc[1][0];
    if (in.sq) {
        ss = wave_sum_bcast(ss);
        if (l == 0) red[w] = ss;
        sync();
        const float r = 1.f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) * in.inv_n + in.eps);
        v0 *= r;
        v1 *= r;
    }
    float s = 0.f;
    if (PAIR) {
        if (l == 0 && row0 < N) e(v0, v1, 0, row0);
    } else if (l < 2 && row0 + l < N) {
        s = e(l ? v1 : v0, 0, row0 + l, int(blockIdx.z));
    }
    if (E::SUMSQ) {
        s += shfl_xor(s, 1);
        if (l == 0) red[4 + w] = s;
        sync();
        if (t == 0) e.sums[blockIdx.x] = (red[4] + red[5]) + (red[6] + red[7]);
    }
}
// 2 .. 16 tokens: a workgroup per 16 RG weight rows, its NW waves on interleaved 128-column blocks of the reduction.  Tokens are the
// rows of A, weight rows the columns of B: both k-contiguous in memory, so fragments come straight from global memory, and the matrix pipe takes the
// multiply-adds of all tokens at the price of one.  RG = 2 reads the tokens once for 32 weight rows: at 16 tokens they are as many bytes as 16 rows;
// PAIR: the second 16 are the up rows of the same outputs.
// (Plain loads: a fragment touches half a cache line of 16 rows and the next one the other half, which a non-temporal hint fetches twice -- 157
// against 123 us for a 514 MB head at 8 tokens.)
template <int NW, int RG, class E, bool PAIR>
__global__ __launch_bounds__(NW * 64) void rows_kernel(RowsPair rp, int n_tok, E e) {
    static_assert(!PAIR || RG == 2, "gate rows beside up rows");
    ARIA_SMEM_STATIC float red[NW][16][16 * RG + 1];
    ARIA_SMEM_STATIC float rms[16];
    const RowsIn& in = rp.in[blockIdx.z];
    const int t = threadIdx.x, l = t & 63, w = t >> 6, q4 = l >> 4, c16 = l & 15, K = in.K, N = in.N;
    constexpr int OUT = PAIR ? 16 : 16 * RG;
    const int n0 = blockIdx.x * OUT, t0 = blockIdx.y * 16;
    const bf16_t* wp[RG];
#pragma unroll
    for (int g = 0; g < RG; ++g) wp[g] = (PAIR && g ? in.W2 : in.W) + (long long)min(n0 + (PAIR ? 0 : 16 * g) + c16, N - 1) * K;
    const bf16_t* xp = in.X + (long long)min(t0 + c16, n_tok - 1) * in.ldx;
    f32x4 acc[RG][2];
#pragma unroll
    for (int g = 0; g < RG; ++g) acc[g][0] = acc[g][1] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int k0 = w * 128; k0 < K; k0 += 2 * NW * 128) {   // two blocks in flight: every weight fragment before the first use
        u32x4 a[8], b[RG][8];
#pragma unroll
        for (int g = 0; g < RG; ++g)
#pragma unroll
            for (int u = 0; u < 8; ++u) {
                const int k = k0 + (u >> 2) * NW * 128 + (u & 3) * 32 + q4 * 8;
                b[g][u] = ld16(wp[g] + (k < K ? k : 0));
            }
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            const int k = k0 + (u >> 2) * NW * 128 + (u & 3) * 32 + q4 * 8;
            a[u] = ld16(xp + (k < K ? k : 0));
#pragma unroll
            for (int q = 0; q < 4; ++q) a[u][q] = k < K ? a[u][q] : 0u;
        }
#pragma unroll
        for (int u = 0; u < 8; ++u)
#pragma unroll
            for (int g = 0; g < RG; ++g) acc[g][u & 1] = mfma16(__builtin_bit_cast(s16x8, a[u]), __builtin_bit_cast(s16x8, b[g][u]), acc[g][u & 1]);
    }
    if (in.sq) {   // 1 / rms of the tokens, a wave per token
        for (int i = w; i < 16 && t0 + i < n_tok; i += NW) {
            float s = 0.f;
            for (int j = l; j < in.sq_n; j += 64) s += in.sq[(long long)(t0 + i) * in.sq_n + j];
            s = wave_sum_bcast(s);
            if (l == 0) rms[i] = 1.f / sqrtf(s * in.inv_n + in.eps);
        }
    }
#pragma unroll
    for (int g = 0; g < RG; ++g)
#pragma unroll
        for (int r = 0; r < 4; ++r) red[w][4 * q4 + r][16 * g + c16] = acc[g][0][r] + acc[g][1][r];
    sync();
    for (int i = t; i < 16 * OUT; i += NW * 64) {   // (whole waves: 16 OUT is a multiple of 64)
        const int tok = i / OUT, n = i % OUT;
        const bool in_range = t0 + tok < n_tok && n0 + n < N;
        float v = 0.f, u = 0.f;
#pragma unroll
        for (int ww = 0; ww < NW; ++ww) {
            v += red[ww][tok][n];
            if (PAIR) u += red[ww][tok][16 + n];
        }
        if (in.sq && in_range) {
            v *= rms[tok];
            u *= rms[tok];
        }
        float s = 0.f;
        if (in_range) {
            if (PAIR)
                e(v, u, t0 + tok, n0 + n);
            else
                s = e(v, t0 + tok, n0 + n, int(blockIdx.z));
        }
        if (E::SUMSQ) {
            static_assert(!E::SUMSQ || OUT == 16, "sixteen lanes hold a token's outputs");
            s = group_sum<16>(s);
            if (n == 0 && t0 + tok < n_tok) e.sums[(long long)(t0 + tok) * gridDim.x + blockIdx.x] = s;
        }
    }
}

// workgroups of one problem, i.e. the partial sums per token that an epilogue with SUMSQ leaves
inline int rows_parts(int64_t T, int64_t N) { return int(T == 1 ? (N + 7) / 8 : (N + 15) / 16); }

template <class E>
int launch_rows(const RowsPair& rp, int problems, int64_t T, const E& e, void* stream) {
    const int64_t N = rp.in[0].N;
    const unsigned z = unsigned(problems), groups = unsigned((T + 15) / 16);
    if constexpr (!E::SUMSQ) {
        if (T > 1 && N > 16 * 1024) {
            ARIA_LAUNCH((rows_kernel<4, 2, E, false>), dim3(unsigned((N + 31) / 32), groups, z), dim3(256), 0, stream, rp, int(T), e);
            return aria_check_launch();
        }
    }
    if (T == 1)
        ARIA_LAUNCH((row_kernel<E, false>), dim3(unsigned((N + 7) / 8), 1, z), dim3(256), 0, stream, rp, e);
    else   // few row groups: more waves per group
        ARIA_LAUNCH((rows_kernel<8, 1, E, false>), dim3(unsigned((N + 15) / 16), groups, z), dim3(512), 0, stream, rp, int(T), e);
    return aria_check_launch();
}
// gated pair: outputs e(gate, up, token, row)
template <class E>
int launch_row_pairs(const RowsIn& in, int64_t T, const E& e, void* stream) {
    const RowsPair rp{{in, in}};
    if (T == 1)
        ARIA_LAUNCH((row_kernel<E, true>), dim3(unsigned((in.N + 3) / 4)), dim3(256), 0, stream, rp, e);
    else
        ARIA_LAUNCH((rows_kernel<8, 2, E, true>), dim3(unsigned((in.N + 15) / 16), unsigned((T + 15) / 16)), dim3(512), 0, stream, rp, int(T), e);
    return aria_check_launch();
}

}  // namespace
}  // namespace ad
