// Linear attention: per head a matrix state S [d, dv] that decays, S_t = diag(a_t) S_(t-1) + k_t v_t^T, and is read by the query, o_t = S_t^T q_t.  The
// decay is one constant per head, or comes per token and key channel from a low-rank projection, a = sigmoid(a2 a1 + b)^(1 / tau).  States are fp32
// and live in the sequence's cache slot; a sequence at position 0 starts from zeros whatever the slot holds.
#include "linear_step.h"
#include "tile.h"

namespace {
using namespace ad;
typedef AriaLinearShape Lin;

bool al16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

// ---------------------------------------------------------------------------------------------- prompts on the matrix pipe (bf16)
// A sequence is cut into blocks of 64 rows.  With G the running sum of the log decays inside a block and a reference R per channel (the middle of the
// block's range), a block needs q^ = q e^(G - R), k^ = k e^(R - G) and the factors e^R, e^(G_last - R) per channel:
//   o = q^ (e^R S) + tril(q^ k^T) v,      S' = e^(G_last - R) (e^R S + k^T v)
// so every product is a matrix product.  linear_prepare writes q^ and k^ in place of q and k.  The exponents stay inside +- RANGE / 2; a block whose
// decay exceeds RANGE (a state that forgets everything within the block) is marked and runs token by token instead.
// Blocks of a sequence form chunks that run side by side: chunk states from zero (linear_chunk_kernel<OUT = false>), a scan over the chunks
// (linear_scan_kernel), then the outputs from each chunk's true first state (OUT = true).
constexpr int BLK = 64;
constexpr float RANGE = 216.f;   // in powers of two: +- 2^108 leaves fp32 and bf16 room for the sums
__device__ const uint32_t linear_zero_page[4] = {};

template <int DP>
__global__ __launch_bounds__(256) void linear_prepare_kernel(bf16_t* proj, Lin s, const int32_t* blocks, float* fac, int32_t* marked, float* alpha) {
    constexpr int PAIRS = DP / 2, NG = 256 / PAIRS, PER = BLK / NG;   // a thread: two channels of PER tokens
    ARIA_DYN_SMEM(smem);
    float* sG = reinterpret_cast<float*>(smem);   // [BLK][DP]
    float* sT = sG + BLK * DP;                    // [NG][DP]
    float* sM = sT + NG * DP;                     // [4]
    float* sA = sM + 4;                           // [BLK][rank]
    const int t = threadIdx.x, l = t & 63, w = t >> 6, d = 2 * (t % PAIRS), grp = t / PAIRS, h = blockIdx.y;
    const int row0 = blocks[2 * blockIdx.x], n = blocks[2 * blockIdx.x + 1], rank = int(s.rank);
    if (!s.decay) {
        for (int i = t; i < BLK * rank; i += 256) {
            const int tok = i / rank;
            sA[i] = tok < n ? ldf(proj + (long long)(row0 + tok) * s.ldp + s.a_off + i % rank) : 0.f;
        }
        sync();
    }
    float z[PER][2];   // log2 of the decay
    if (s.decay) {
        const float v = s.decay[2 * h + 1];
#pragma unroll
        for (int i = 0; i < PER; ++i) z[i][0] = z[i][1] = v;
    } else {
        const long long ch = (long long)h * DP + d;
        const bf16_t* a2 = static_cast<const bf16_t*>(s.a2) + ch * rank;
        const float b0 = s.a_bias[ch], b1 = s.a_bias[ch + 1];
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            z[i][0] = b0;
            z[i][1] = b1;
        }
        for (int r = 0; r < rank; r += 8) {
            float w0[8], w1[8];
            ld8(a2 + r, w0);
            ld8(a2 + rank + r, w1);
#pragma unroll
            for (int i = 0; i < PER; ++i) {
                float a[8];
                ld8(sA + (grp * PER + i) * rank + r, a);
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    z[i][0] += w0[e] * a[e];
                    z[i][1] += w1[e] * a[e];
                }
            }
        }
#pragma unroll
        for (int i = 0; i < PER; ++i)
#pragma unroll
            for (int c = 0; c < 2; ++c) z[i][c] = (fminf(z[i][c], 0.f) - log1pf(expf(-fabsf(z[i][c])))) * s.inv_tau * 1.4426950408889634f;
    }
    float c0 = 0.f, c1 = 0.f;
#pragma unroll
    for (int i = 0; i < PER; ++i) {
        const int tok = grp * PER + i;
        if (tok < n) {
            c0 += z[i][0];
            c1 += z[i][1];
        }
        sG[tok * DP + d] = c0;
        sG[tok * DP + d + 1] = c1;
    }
    sT[grp * DP + d] = c0;
    sT[grp * DP + d + 1] = c1;
    sync();
    float o0 = 0.f, o1 = 0.f, last0 = 0.f, last1 = 0.f;
#pragma unroll
    for (int g = 0; g < NG; ++g) {
        if (g == grp) o0 = last0, o1 = last1;
        last0 += sT[g * DP + d];
        last1 += sT[g * DP + d + 1];
    }
    const float first0 = sG[d], first1 = sG[d + 1];
    float drop = fmaxf(first0 - last0, first1 - last1);
    if (!(first0 - last0 <= RANGE) || !(first1 - last1 <= RANGE)) drop = INFINITY;   // (not a number: a decay of zero)
    drop = wave_max_bcast(drop);
    if (l == 0) sM[w] = drop;
    sync();
    const bool exact = !(fmaxf(fmaxf(sM[0], sM[1]), fmaxf(sM[2], sM[3])) <= RANGE);
    const long long bh = (long long)blockIdx.x * s.H + h;
    if (t == 0) marked[bh] = exact;
    const float R0 = 0.5f * (first0 + last0), R1 = 0.5f * (first1 + last1);
    if (grp == 0) {
        float* f = fac + bh * 3 * DP + d;
        f[0] = exp2f(R0);
        f[1] = exp2f(R1);
        f[DP] = exp2f(last0 - R0);
        f[DP + 1] = exp2f(last1 - R1);
        f[2 * DP] = exp2f(last0);
        f[2 * DP + 1] = exp2f(last1);
    }
#pragma unroll
    for (int i = 0; i < PER; ++i) {
        const int tok = grp * PER + i;
        if (tok >= n) continue;
        bf16_t* p = proj + (long long)(row0 + tok) * s.ldp + h * DP + d;
        const uint32_t qw = *reinterpret_cast<const uint32_t*>(p + s.q_off), kw = *reinterpret_cast<const uint32_t*>(p + s.k_off);
        float q0 = bflo(qw), q1 = bfhi(qw), k0 = bflo(kw), k1 = bfhi(kw);
        if (s.silu) q0 = silu_fast(q0), q1 = silu_fast(q1), k0 = silu_fast(k0), k1 = silu_fast(k1);
        q0 *= s.q_scale;
        q1 *= s.q_scale;
        if (exact) {
            float* a = alpha + ((long long)(row0 + tok) * s.H + h) * DP + d;
            a[0] = exp2f(z[i][0]);
            a[1] = exp2f(z[i][1]);
        } else {
            const float e0 = sG[tok * DP + d] + o0 - R0, e1 = sG[tok * DP + d + 1] + o1 - R1;
            q0 *= exp2f(e0);
            q1 *= exp2f(e1);
            k0 *= exp2f(-e0);
            k1 *= exp2f(-e1);
        }
        *reinterpret_cast<uint32_t*>(p + s.q_off) = pack2bf(q0, q1);
        *reinterpret_cast<uint32_t*>(p + s.k_off) = pack2bf(k0, k1);
    }
    if (s.silu) {
        const int vc = int(s.dvp) >> 3;
        for (int i = t; i < n * vc; i += 256) {
            bf16_t* p = proj + (long long)(row0 + i / vc) * s.ldp + s.v_off + h * s.dvp + (i % vc) * 8;
            float v[8];
            ld8(p, v);
#pragma unroll
            for (int e = 0; e < 8; ++e) v[e] = silu_fast(v[e]);
            st8(p, v);
        }
    }
}

// grid (32 NW-column blocks of the values, heads, chunks), NW waves.  Wave w holds the state's columns 32 w .. + 31 for all DP channels as 32 x 32
// accumulators [channel][column]; read as the A operand of o^T = S^T q^T their registers are in place (the channel order inside a 16-block follows the
// accumulator, q^ is read in that order).  The state enters that product as two bf16 numbers, so it is read with 16 bits of mantissa.
// LDS: q^ and k^ images, v image, scores [64][PP], factors.  Per block three barriers: q^ arrives while the previous block's state is updated, k^ and v
// while S^T q^T runs.
template <int DP, int NW>
struct ChunkSmem {
    static constexpr int VB = 32 * NW, PP = 72;
    static constexpr int Q0 = 0, K0 = TileImg<DP>::BYTES, V0 = 2 * K0, P0 = V0 + TileImg<VB>::BYTES, F0 = P0 + 64 * PP * 2, BYTES = F0 + 2 * 2 * DP * 4;
};
template <int DP, int NW, bool OUT>
__global__ __launch_bounds__(NW * 64) void linear_chunk_kernel(const bf16_t* proj, Lin s, const int32_t* blocks, const int32_t* chunks, const float* fac,
                                                               const int32_t* marked, const float* alpha, float* states, float* cache, const int32_t* slot,
                                                               const int32_t* pos, bf16_t* out) {
    using L = ChunkSmem<DP, NW>;
    using QI = TileImg<DP>;
    using VI = TileImg<L::VB>;
    constexpr int TD = DP / 32, KV_PIECES = DP / 8 / NW + 4;
    ARIA_DYN_SMEM(smem);
    char *sQ = smem + L::Q0, *sK = smem + L::K0, *sV = smem + L::V0;
    bf16_t* sP = reinterpret_cast<bf16_t*>(smem + L::P0);
    float* sF = reinterpret_cast<float*>(smem + L::F0);   // [2][2 DP]
    const int t = threadIdx.x, l = t & 63, w = first_lane(t >> 6), h2 = l >> 5, c32 = l & 31, q4 = l >> 4, c16 = l & 15;
    const int v0 = blockIdx.x * L::VB, h = blockIdx.y, c = blockIdx.z;
    const int b0 = chunks[4 * c], nb = chunks[4 * c + 1], first = chunks[4 * c + 2], last = chunks[4 * c + 3];
    if (!OUT && last) return;
    const int vcol = v0 + 32 * w;            // this wave's first column
    const bool mine = vcol < s.dvp;
    const long long head_state = (long long)s.dp * s.dvp, H = s.H;
    const int r_first = blocks[2 * b0];
    float* slot_state = cache + ((long long)slot[r_first] * H + h) * head_state + vcol + c32;
    f32x16 S[TD];
#pragma unroll
    for (int i = 0; i < TD; ++i) S[i] = zero_acc();
    const bool alone = first && last;        // the chunk is its whole sequence: from the cache into the cache
    if (OUT && mine && !(alone && pos[r_first] == 0)) {
        const float* src = alone ? slot_state : states + ((long long)c * H + h) * head_state + vcol + c32;
#pragma unroll
        for (int i = 0; i < TD; ++i)
#pragma unroll
            for (int r = 0; r < 16; ++r) S[i][r] = src[(long long)(32 * i + acc_row(r, l)) * s.dvp];
    }
    auto dma_rows = [&](const bf16_t* base, int n, char* dst) __attribute__((always_inline)) {   // q^ or k^: DP columns
#pragma unroll
        for (int i = 0; i < DP / 8 / NW; ++i) {
            const int pc = w + NW * i, ch = pc * 64 + l, row = ch / QI::CPR, col = ((ch % QI::CPR) ^ QI::swz(row)) * 8;
            const void* src = row < n ? static_cast<const void*>(base + (long long)row * s.ldp + col) : static_cast<const void*>(linear_zero_page);
            glds16_raw(src, dst + pc * 1024);
        }
    };
    auto dma_q = [&](int b) __attribute__((always_inline)) {
        dma_rows(proj + (long long)blocks[2 * b] * s.ldp + s.q_off + h * DP, blocks[2 * b + 1], sQ);
    };
    auto dma_kv = [&](int b) __attribute__((always_inline)) {
        const int n = blocks[2 * b + 1];
        const bf16_t* rows = proj + (long long)blocks[2 * b] * s.ldp;
        dma_rows(rows + s.k_off + h * DP, n, sK);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int pc = w + NW * i, ch = pc * 64 + l, row = ch / VI::CPR, col = v0 + ((ch % VI::CPR) ^ VI::swz(row)) * 8;
            const void* src = row < n && col < s.dvp ? static_cast<const void*>(rows + (long long)row * s.ldp + s.v_off + h * s.dvp + col)
                                                     : static_cast<const void*>(linear_zero_page);
            glds16_raw(src, sV + pc * 1024);
        }
    };
    auto barrier = [&]() __attribute__((always_inline)) {   // (LDS-DMA in flight stays in flight)
        wait_lds();
        raw_barrier();
    };
    f32x4 fnext = f32x4{0.f, 0.f, 0.f, 0.f};
    auto fetch_f = [&](int b) __attribute__((always_inline)) {
        if (t < DP / 2) fnext = *reinterpret_cast<const f32x4*>(fac + ((long long)b * H + h) * 3 * DP + 4 * t);
    };
    auto park_f = [&](int buf) __attribute__((always_inline)) {
        if (t < DP / 2) *reinterpret_cast<f32x4*>(sF + buf * 2 * DP + 4 * t) = fnext;
    };
    auto scale_rows = [&](f32x16& x, const float* f, int td) __attribute__((always_inline)) {
#pragma unroll
        for (int rg = 0; rg < 4; ++rg) {
            const f32x4 v = *reinterpret_cast<const f32x4*>(f + 32 * td + 8 * rg + 4 * h2);
#pragma unroll
            for (int e = 0; e < 4; ++e) x[4 * rg + e] *= v[e];
        }
    };
    fetch_f(b0);
    if (OUT) {
        for (int i = t; i < 64 * L::PP / 8; i += NW * 64) st16(sP + i * 8, zero16());   // (tiles above the diagonal stay zero)
        dma_q(b0);
    }
    dma_kv(b0);
    park_f(0);
    for (int j = 0; j < nb; ++j) {
        const int b = b0 + j, row0 = blocks[2 * b], n = blocks[2 * b + 1];
        const float* f = sF + (j & 1) * 2 * DP;
        const bool more = j + 1 < nb;
        if (marked[(long long)b * H + h]) {   // (workgroup-uniform) token by token: decays from alpha, q, k, v as they lie in proj
            for (int i = 0; i < n; ++i) {
                const bf16_t* p = proj + (long long)(row0 + i) * s.ldp;
                const float* a = alpha + ((long long)(row0 + i) * H + h) * DP;
                const float v = mine ? ldf(p + s.v_off + h * s.dvp + vcol + c32) : 0.f;
                float o = 0.f;
#pragma unroll
                for (int td = 0; td < TD; ++td)
#pragma unroll
                    for (int r = 0; r < 16; ++r) {
                        const int d = 32 * td + acc_row(r, l);
                        S[td][r] = a[d] * S[td][r] + ldf(p + s.k_off + h * DP + d) * v;
                        if (OUT) o += S[td][r] * ldf(p + s.q_off + h * DP + d);
                    }
                if (OUT) {
                    o += shfl_xor(o, 32);
                    if (mine && h2 == 0) stf(out + ((long long)(row0 + i) * H + h) * s.dvp + vcol + c32, o);
                }
            }
            wait_vm<0>();
            barrier();
            if (more) {
                fetch_f(b + 1);
                if (OUT) dma_q(b + 1);
                dma_kv(b + 1);
                park_f((j + 1) & 1);
            }
            continue;
        }
        f32x16 o[2];
        if (OUT) {
            wait_vm<KV_PIECES>();   // q^ has landed (k^ and v, requested after it, may be in flight)
            barrier();
            o[0] = zero_acc();
            o[1] = zero_acc();
#pragma unroll
            for (int td = 0; td < TD; ++td) {
                scale_rows(S[td], f, td);
#pragma unroll
                for (int u = 0; u < 2; ++u) {
                    const s16x8 hi = pack_frag(S[td], u);
                    f32x16 rest;
#pragma unroll
                    for (int e = 0; e < 8; ++e) rest[8 * u + e] = S[td][8 * u + e] - bf2f(bf16_t(hi[e]));
                    const s16x8 lo = pack_frag(rest, u);
                    const int ch = (32 * td + 16 * u) >> 3;
#pragma unroll
                    for (int tt = 0; tt < 2; ++tt) {
                        const int row = 32 * tt + c32;
                        const char* base = sQ + row * QI::ROW + 8 * h2;
                        const s16x4 x0 = *reinterpret_cast<const s16x4*>(base + ((ch ^ QI::swz(row)) << 4));
                        const s16x4 x1 = *reinterpret_cast<const s16x4*>(base + (((ch + 1) ^ QI::swz(row)) << 4));
                        s16x8 qf;
#pragma unroll
                        for (int e = 0; e < 4; ++e) {
                            qf[e] = x0[e];
                            qf[4 + e] = x1[e];
                        }
                        o[tt] = mfma32(hi, qf, o[tt]);
                        o[tt] = mfma32(lo, qf, o[tt]);
                    }
                }
            }
        }
        wait_vm<0>();
        barrier();
        if (OUT) {   // scores: 16 x 16 tiles (a, b) of the lower triangle, rows = keys 4 q4 + r, columns = queries
            for (int x = w; x < 10; x += NW) {
                const int a = x < 1 ? 0 : x < 3 ? 1 : x < 6 ? 2 : 3, kb = x - a * (a + 1) / 2;
                f32x4 sc[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
                const int kr = 16 * kb + c16, qr = 16 * a + c16;
#pragma unroll
                for (int kk = 0; kk < DP / 32; ++kk) {
                    const s16x8 ka = *reinterpret_cast<const s16x8*>(sK + kr * QI::ROW + (((4 * kk + q4) ^ QI::swz(kr)) << 4));
                    const s16x8 qb = *reinterpret_cast<const s16x8*>(sQ + qr * QI::ROW + (((4 * kk + q4) ^ QI::swz(qr)) << 4));
                    sc[kk & 1] = mfma16(ka, qb, sc[kk & 1]);
                }
                float p[4];
#pragma unroll
                for (int r = 0; r < 4; ++r) p[r] = a == kb && 4 * q4 + r > c16 ? 0.f : sc[0][r] + sc[1][r];
                *reinterpret_cast<u32x2*>(sP + qr * L::PP + 16 * kb + 4 * q4) = u32x2{pack2bf(p[0], p[1]), pack2bf(p[2], p[3])};
            }
            barrier();   // scores complete; every wave is done with q^
            if (more) dma_q(b + 1);
        }
        if (more) fetch_f(b + 1);
        s16x8 vf[4];
#pragma unroll
        for (int jb = 0; jb < 4; ++jb) vf[jb] = VI::columns(sV, 16 * jb, 32 * w, l);
        if (OUT) {
#pragma unroll
            for (int tt = 0; tt < 2; ++tt)
#pragma unroll
                for (int jb = 0; jb < 2 + 2 * tt; ++jb) {
                    const bf16_t* src = sP + (32 * tt + c32) * L::PP + 16 * jb + 4 * h2;
                    const s16x4 x0 = *reinterpret_cast<const s16x4*>(src), x1 = *reinterpret_cast<const s16x4*>(src + 8);
                    s16x8 pf;
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        pf[e] = x0[e];
                        pf[4 + e] = x1[e];
                    }
                    o[tt] = mfma32(vf[jb], pf, o[tt]);
                }
#pragma unroll
            for (int tt = 0; tt < 2; ++tt)
                if (mine && 32 * tt + c32 < n) {
                    bf16_t* dst = out + ((long long)(row0 + 32 * tt + c32) * H + h) * s.dvp + vcol + 4 * h2;
#pragma unroll
                    for (int rg = 0; rg < 4; ++rg)
                        *reinterpret_cast<u32x2*>(dst + 8 * rg) =
                            u32x2{pack2bf(o[tt][4 * rg], o[tt][4 * rg + 1]), pack2bf(o[tt][4 * rg + 2], o[tt][4 * rg + 3])};
                }
        }
#pragma unroll
        for (int td = 0; td < TD; ++td) {
            if (!OUT) scale_rows(S[td], f, td);
#pragma unroll
            for (int jb = 0; jb < 4; ++jb) S[td] = mfma32(QI::columns(sK, 16 * jb, 32 * td, l), vf[jb], S[td]);
            scale_rows(S[td], f + DP, td);
        }
        if (more) park_f((j + 1) & 1);
        barrier();   // every wave is done with k^, v and (OUT = false) the factors' other half
        if (more) dma_kv(b + 1);
    }
    if (!mine || (OUT && !last)) return;
    float* dst = OUT ? slot_state : states + ((long long)(c + 1) * H + h) * head_state + vcol + c32;
#pragma unroll
    for (int i = 0; i < TD; ++i)
#pragma unroll
        for (int r = 0; r < 16; ++r) dst[(long long)(32 * i + acc_row(r, l)) * s.dvp] = S[i][r];
}

// first states of the chunks: states[c] holds chunk c - 1's state from zero; on return the state in front of chunk c.  A thread: four columns of one
// channel, all chunks of a sequence.
__global__ __launch_bounds__(256) void linear_scan_kernel(Lin s, const int32_t* blocks, const int32_t* chunks, const int32_t* seqs, const float* fac, float* states,
                                                          const float* cache, const int32_t* slot, const int32_t* pos) {
    const int i = blockIdx.x * 256 + threadIdx.x, h = blockIdx.y, c0 = seqs[2 * blockIdx.z], nc = seqs[2 * blockIdx.z + 1];
    const long long head_state = s.dp * s.dvp, H = s.H;
    if (nc < 2 || 4ll * i >= head_state) return;
    const int d = int(4ll * i / s.dvp), r0 = blocks[2 * chunks[4 * c0]];
    f32x4 x = f32x4{0.f, 0.f, 0.f, 0.f};
    if (pos[r0] > 0) x = *reinterpret_cast<const f32x4*>(cache + ((long long)slot[r0] * H + h) * head_state + 4 * i);
    float* at = states + ((long long)c0 * H + h) * head_state + 4 * i;
    *reinterpret_cast<f32x4*>(at) = x;
    for (int c = c0; c + 1 < c0 + nc; ++c) {
        at += H * head_state;
        const f32x4 own = *reinterpret_cast<const f32x4*>(at);
        float a = 1.f;
        const int b0 = chunks[4 * c], nb = chunks[4 * c + 1];
        for (int b = b0; b < b0 + nb; ++b) a *= fac[(((long long)b * H + h) * 3 + 2) * s.dp + d];
#pragma unroll
        for (int e = 0; e < 4; ++e) x[e] = a * x[e] + own[e];
        *reinterpret_cast<f32x4*>(at) = x;
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

struct ChunkScratch {
    float *fac, *alpha, *states;
    int32_t* marked;
    int64_t bytes;
};
ChunkScratch layout(const Lin& s, int64_t T, int64_t n_blocks, int64_t n_chunks, char* base) {
    ChunkScratch z{};
    int64_t at = 0;
    auto take = [&](int64_t bytes) {
        char* p = base + at;
        at += (bytes + 255) & ~int64_t(255);
        return p;
    };
    z.fac = reinterpret_cast<float*>(take(4 * n_blocks * s.H * 3 * s.dp));
    z.marked = reinterpret_cast<int32_t*>(take(4 * n_blocks * s.H));
    z.alpha = reinterpret_cast<float*>(take(4 * T * s.H * s.dp));
    z.states = reinterpret_cast<float*>(take(4 * n_chunks * s.H * s.dp * s.dvp));
    z.bytes = at;
    return z;
}

struct ChunkArgs {
    bf16_t* proj;
    const Lin& s;
    float* state;
    const int32_t *slot, *pos, *blocks, *chunks, *seqs;
    int64_t n_blocks, n_chunks, n_seq;
    bf16_t* out;
    ChunkScratch z;
    void* stream;
};
template <int DP, int NW>
int launch_chunks(const ChunkArgs& a) {
    using L = ChunkSmem<DP, NW>;
    const Lin& s = a.s;
    const dim3 grid(unsigned((s.dvp + L::VB - 1) / L::VB), unsigned(s.H), unsigned(a.n_chunks)), block(NW * 64);
    if (a.n_chunks > a.n_seq) {
        ARIA_LAUNCH((linear_chunk_kernel<DP, NW, false>), grid, block, size_t(L::BYTES), a.stream, (const bf16_t*)a.proj, s, a.blocks, a.chunks,
                    (const float*)a.z.fac, (const int32_t*)a.z.marked, (const float*)a.z.alpha, a.z.states, a.state, a.slot, a.pos, a.out);
        const int64_t n4 = s.dp * s.dvp / 4;
        ARIA_LAUNCH(linear_scan_kernel, dim3(unsigned((n4 + 255) / 256), unsigned(s.H), unsigned(a.n_seq)), dim3(256), 0, a.stream, s, a.blocks, a.chunks,
                    a.seqs, (const float*)a.z.fac, a.z.states, (const float*)a.state, a.slot, a.pos);
    }
    ARIA_LAUNCH((linear_chunk_kernel<DP, NW, true>), grid, block, size_t(L::BYTES), a.stream, (const bf16_t*)a.proj, s, a.blocks, a.chunks, (const float*)a.z.fac,
                (const int32_t*)a.z.marked, (const float*)a.z.alpha, a.z.states, a.state, a.slot, a.pos, a.out);
    return aria_check_launch();
}
template <int DP>
int run_chunks(const ChunkArgs& a) {
    const size_t lds = size_t(BLK * DP + (256 / (DP / 2)) * DP + 4 + BLK * a.s.rank) * 4;
    if (lds > 160 * 1024) return ARIA_ERR_UNSUPPORTED;
    ARIA_LAUNCH((linear_prepare_kernel<DP>), dim3(unsigned(a.n_blocks), unsigned(a.s.H)), dim3(256), lds, a.stream, a.proj, a.s, a.blocks, a.z.fac, a.z.marked,
                a.z.alpha);
    return a.s.dvp <= 64 ? launch_chunks<DP, 2>(a) : launch_chunks<DP, 4>(a);
}

}  // namespace

extern "C" {

int64_t aria_linear_chunks_scratch(const AriaLinearShape* s, int64_t T, int64_t n_blocks, int64_t n_chunks) {
    return s && T > 0 ? layout(*s, T, n_blocks, n_chunks, nullptr).bytes : 0;
}

int aria_linear_chunks(void* proj, const AriaLinearShape* s, float* state, const int32_t* slot, const int32_t* pos, const int32_t* blocks, int64_t n_blocks,
                       const int32_t* chunks, int64_t n_chunks, const int32_t* seqs, int64_t n_seq, void* out, int64_t T, void* scratch,
                       int64_t scratch_bytes, void* stream) {
    if (!proj || !state || !slot || !pos || !blocks || !chunks || !seqs || !out || !scratch || T < 0 || n_blocks < 0 || n_chunks < n_seq || n_seq < 0)
        return ARIA_ERR_INVALID;
    if (const int rc = shape_ok(s)) return rc;
    if (!al16(proj) || !al16(state) || !al16(out) || !al16(scratch)) return ARIA_ERR_ALIGN;
    if ((s->dvp & 63) || n_chunks > 65535 || s->H > 65535) return ARIA_ERR_UNSUPPORTED;
    if (T == 0 || n_seq == 0) return ARIA_OK;
    const ChunkArgs a{static_cast<bf16_t*>(proj), *s, state, slot, pos, blocks, chunks, seqs, n_blocks, n_chunks, n_seq, static_cast<bf16_t*>(out),
                      layout(*s, T, n_blocks, n_chunks, static_cast<char*>(scratch)), stream};
    if (scratch_bytes < a.z.bytes) return ARIA_ERR_INVALID;
    switch (s->dp) {
        case 64: return run_chunks<64>(a);
        case 128: return run_chunks<128>(a);
        case 256: return run_chunks<256>(a);
    }
    return ARIA_ERR_UNSUPPORTED;
}

int aria_linear_step(const void* proj, const AriaLinearShape* s, float* state, const int32_t* slot, const int32_t* pos, const int32_t* cu, int64_t n_seq,
                     void* out, int f32, void* stream) {
    if (!proj || !state || !slot || !pos || !cu || !out || n_seq < 0) return ARIA_ERR_INVALID;
    if (const int rc = shape_ok(s)) return rc;
    if (!al16(proj) || !al16(state)) return ARIA_ERR_ALIGN;
    if (s->dp > 1024 || s->H > 65535 || n_seq > 65535) return ARIA_ERR_UNSUPPORTED;
    if (n_seq == 0) return ARIA_OK;
    const StepOut plain{};
    return f32 ? launch_step<float>(proj, *s, state, slot, pos, cu, n_seq, out, plain, stream)
               : launch_step<bf16_t>(proj, *s, state, slot, pos, cu, n_seq, out, plain, stream);
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
