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

constexpr int PREP = 512;   // threads of linear_prepare
template <int DP>
__global__ __launch_bounds__(PREP) void linear_prepare_kernel(bf16_t* proj, Lin s, const int32_t* blocks, float* fac, int32_t* marked, float* alpha) {
    constexpr int PAIRS = DP / 2, NG = PREP / PAIRS, PER = BLK / NG;   // a thread: two channels of PER tokens
    ARIA_DYN_SMEM(smem);
    float* sT = reinterpret_cast<float*>(smem);   // [NG + 1][DP]: the groups' sums, the first token's value
    float* sM = sT + (NG + 1) * DP;               // [8]
    float* sA = sM + 8;                           // [BLK][rank]
    const int t = threadIdx.x, l = t & 63, w = t >> 6, d = 2 * (t % PAIRS), grp = t / PAIRS, h = blockIdx.y;
    const int row0 = blocks[2 * blockIdx.x], n = blocks[2 * blockIdx.x + 1], rank = int(s.rank);
    if (!s.decay) {
        for (int i = t; i < BLK * rank; i += PREP) {
            const int tok = i / rank;
            sA[i] = tok < n ? ldf(proj + (long long)(row0 + tok) * s.ldp + s.a_off + i % rank) : 0.f;
        }
        sync();
    }
    // this thread's queries and keys, requested before anything is computed (the stores below go to the same rows)
    uint32_t qw[PER], kw[PER];
#pragma unroll
    for (int i = 0; i < PER; ++i) {
        const bf16_t* p = proj + (long long)(row0 + min(grp * PER + i, n - 1)) * s.ldp + h * DP + d;
        qw[i] = *reinterpret_cast<const uint32_t*>(p + s.q_off);
        kw[i] = *reinterpret_cast<const uint32_t*>(p + s.k_off);
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
            for (int c = 0; c < 2; ++c) z[i][c] = log2_sigmoid_fast(z[i][c]) * s.inv_tau;
    }
    if (grp == 0) {
        sT[NG * DP + d] = z[0][0];
        sT[NG * DP + d + 1] = z[0][1];
    }
#pragma unroll
    for (int i = 0; i < PER; ++i)   // running sums inside the group
#pragma unroll
        for (int c = 0; c < 2; ++c) z[i][c] = (grp * PER + i < n ? z[i][c] : 0.f) + (i ? z[i - 1][c] : 0.f);
    sT[grp * DP + d] = z[PER - 1][0];
    sT[grp * DP + d + 1] = z[PER - 1][1];
    sync();
    float o0 = 0.f, o1 = 0.f, last0 = 0.f, last1 = 0.f;
#pragma unroll
    for (int g = 0; g < NG; ++g) {
        if (g == grp) o0 = last0, o1 = last1;
        last0 += sT[g * DP + d];
        last1 += sT[g * DP + d + 1];
    }
    const float first0 = sT[NG * DP + d], first1 = sT[NG * DP + d + 1];
    float drop = fmaxf(first0 - last0, first1 - last1);
    if (!(first0 - last0 <= RANGE) || !(first1 - last1 <= RANGE)) drop = INFINITY;   // (not a number: a decay of zero)
    drop = wave_max_bcast(drop);
    if (l == 0) sM[w] = drop;
    sync();
    for (int i = 0; i < PREP / 64; ++i) drop = fmaxf(drop, sM[i]);
    const bool exact = !(drop <= RANGE);
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
        float q0 = bflo(qw[i]), q1 = bfhi(qw[i]), k0 = bflo(kw[i]), k1 = bfhi(kw[i]);
        if (s.silu) q0 = silu_fast(q0), q1 = silu_fast(q1), k0 = silu_fast(k0), k1 = silu_fast(k1);
        q0 *= s.q_scale;
        q1 *= s.q_scale;
        if (exact) {
            float* a = alpha + ((long long)(row0 + tok) * s.H + h) * DP + d;
#pragma unroll
            for (int c = 0; c < 2; ++c)
                a[c] = s.decay ? s.decay[2 * h] : exp2f(gate_log2(s, proj + (long long)(row0 + tok) * s.ldp + s.a_off, h * DP + d + c));
        } else {
            const float e0 = z[i][0] + o0 - R0, e1 = z[i][1] + o1 - R1;
            q0 *= exp2_fast(e0);
            q1 *= exp2_fast(e1);
            k0 *= exp2_fast(-e0);
            k1 *= exp2_fast(-e1);
        }
        *reinterpret_cast<uint32_t*>(p + s.q_off) = pack2bf(q0, q1);
        *reinterpret_cast<uint32_t*>(p + s.k_off) = pack2bf(k0, k1);
    }
    if (s.silu) {
        const int vc = int(s.dvp) >> 3;
        for (int i0 = t; i0 < n * vc; i0 += 4 * PREP) {
            u32x4 x[4];
            bf16_t* p[4];
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                const int i = min(i0 + PREP * u, n * vc - 1);
                p[u] = proj + (long long)(row0 + i / vc) * s.ldp + s.v_off + h * s.dvp + (i % vc) * 8;
                x[u] = ld16(p[u]);
            }
#pragma unroll
            for (int u = 0; u < 4; ++u) {
#pragma unroll
                for (int e = 0; e < 4; ++e) x[u][e] = pack2bf(silu_fast(bflo(x[u][e])), silu_fast(bfhi(x[u][e])));
                if (i0 + PREP * u < n * vc) st16(p[u], x[u]);
            }
        }
    }
}

// A workgroup: 32 NW value columns of a head's chunk, NW DS waves.  Wave w holds the state's columns 32 (w % NW) .. + 31 for its 1 / DS of the DP
// channels (DS = 2 for 256: the state's registers) as 32 x 32 accumulators [channel][column]; read as the A operand of o^T = S^T q^T their registers are in place (the channel order inside a 16-block follows the
// accumulator, q^ is read in that order).  The state enters that product as two bf16 numbers, so it is read with 16 bits of mantissa.
// DS = 2: the two waves of a column slice exchange partial sums through LDS, each finishes one half of the block's tokens.
// LDS: images of q^ (two), k^ and v, scores [64][PP], factors, partial sums; OUT = false: two k^ and v images.  Per block three barriers: q^ is requested a
// whole block ahead, k^ and v at the end of the block before; k^ is awaited behind S^T q^T, v behind the scores.
template <int DP, int NW, bool OUT>
struct ChunkSmem {
    static constexpr int DS = DP > 128 ? 2 : 1, WAVES = NW * DS, VB = 32 * NW, PP = 72, QB = TileImg<DP>::BYTES, VBYTES = TileImg<VB>::BYTES;
    static constexpr int Q0 = 0, K0 = OUT ? 2 * QB : 0, K_STEP = OUT ? 0 : QB, V0 = K0 + QB + K_STEP, V_STEP = OUT ? 0 : VBYTES, P0 = V0 + VBYTES + V_STEP,
                         F0 = P0 + (OUT ? 64 * PP * 2 : 0), O0 = F0 + 2 * DP * 4, BYTES = O0 + (OUT && DS == 2 ? WAVES * 4096 : 0);
};
template <int DP, int NW, bool OUT>
__global__ __launch_bounds__(NW * (DP > 128 ? 128 : 64), 2) void linear_chunk_kernel(const bf16_t* proj, Lin s, const int32_t* blocks, const int32_t* chunks, const float* fac,
                                                               const int32_t* marked, const float* alpha, float* states, float* decays, float* cache,
                                                               const int32_t* slot, const int32_t* pos, bf16_t* out, int n_chunks) {
    using L = ChunkSmem<DP, NW, OUT>;
    using QI = TileImg<DP>;
    using VI = TileImg<L::VB>;
    constexpr int DS = L::DS, NWT = L::WAVES, TD = DP / 32 / DS, Q_PIECES = DP / 8 / NWT, V_PIECES = 4 / DS, OT = 2 / DS;   // OT: token halves a wave finishes
    ARIA_DYN_SMEM(smem);
    bf16_t* sP = reinterpret_cast<bf16_t*>(smem + L::P0);
    float* sF = reinterpret_cast<float*>(smem + L::F0);   // [2][DP]
    const int t = threadIdx.x, l = t & 63, w = first_lane(t >> 6), h2 = l >> 5, c32 = l & 31, q4 = l >> 4, c16 = l & 15;
    const int ws = w % NW, ds = DS == 2 ? w / NW : 0, td0 = ds * TD;   // this wave's column slice, channel half
    // workgroup n runs on XCD n % 8: the column blocks of a (head, chunk) share an XCD, whose L2 then holds their q^ and k^
    const int nvb = (int(s.dvp) + L::VB - 1) / L::VB, group = int(blockIdx.x >> 3) / nvb * 8 + int(blockIdx.x & 7), vb = int(blockIdx.x >> 3) % nvb;
    if (group >= int(s.H) * n_chunks) return;
    const int v0 = vb * L::VB, h = group % int(s.H), c = group / int(s.H);
    const int b0 = chunks[4 * c], nb = chunks[4 * c + 1], first = chunks[4 * c + 2], last = chunks[4 * c + 3];
    if (!OUT && last) return;
    const int vcol = v0 + 32 * ws;           // this wave's first column
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
            for (int r = 0; r < 16; ++r) S[i][r] = src[(long long)(32 * (td0 + i) + acc_row(r, l)) * s.dvp];
    }
    // rows of block j of the chunk: r_first + 64 j .., at most 64
    const int rows_all = blocks[2 * (b0 + nb - 1)] + blocks[2 * (b0 + nb - 1) + 1] - r_first;
    unsigned long long marks = 0;            // marked blocks among j & ~63 ..
    auto load_marks = [&](int j) __attribute__((always_inline)) { marks = ballot(j + l < nb && marked[(long long)(b0 + j + l) * H + h] != 0); };
    auto is_marked = [&](int j) __attribute__((always_inline)) -> bool { return (marks >> (j & 63)) & 1; };
    // this lane's chunk of the wave's first DMA piece of an image; later pieces lie a fixed number of rows further on (the swizzle repeats every 16 rows)
    auto dma_image = [&](auto img, const bf16_t* base, int n, int cols, char* dst) __attribute__((always_inline)) {
        using I = decltype(img);
        constexpr int STEP = NWT * 64 / I::CPR;
        static_assert(STEP % 8 == 0, "");
        int lane = w * 64 + l;
        hold(lane);   // (here and below: addresses are cheaper computed again per block than held in registers beside the state)
        const int row = lane / I::CPR, col = ((lane % I::CPR) ^ I::swz(row)) * 8;
        const char* at = reinterpret_cast<const char*>(base + (long long)row * s.ldp + col);
        const char* zero = reinterpret_cast<const char*>(linear_zero_page);
        const long long step = 2ll * STEP * s.ldp;
#pragma unroll
        for (int i = 0; i < 64 / STEP; ++i) {
            const int c = STEP % 16 && i % 2 ? ((lane % I::CPR) ^ I::swz(row + STEP)) * 8 : col;   // (steps of 8 rows: every other piece has another swizzle)
            const char* src = at + i * step + 2 * (c - col);
            const bool in = row + STEP * i < n && c < cols;
            src = in ? src : zero;
            glds16_raw(src, dst + (w + NWT * i) * 1024);
        }
    };
    auto dma_q = [&](int j, int buf) __attribute__((always_inline)) {
        dma_image(QI(), proj + (long long)(r_first + BLK * j) * s.ldp + s.q_off + h * DP, rows_all - BLK * j, DP, smem + L::Q0 + buf * L::QB);
    };
    auto dma_kv = [&](int j, int buf) __attribute__((always_inline)) {   // (buf: OUT = false has two)
        const bf16_t* rows = proj + (long long)(r_first + BLK * j) * s.ldp;
        dma_image(QI(), rows + s.k_off + h * DP, rows_all - BLK * j, DP, smem + L::K0 + buf * L::K_STEP);
        dma_image(VI(), rows + s.v_off + h * s.dvp + v0, rows_all - BLK * j, int(s.dvp) - v0, smem + L::V0 + buf * L::V_STEP);
    };
    auto barrier = [&]() __attribute__((always_inline)) {   // (LDS-DMA in flight stays in flight)
        wait_lds();
        raw_barrier();
    };
    // per-channel factors of a block's start, e^(G_last - R) of the block before times e^R of its own: thread t owns channels 4 t .. 4 t + 3
    const f32x4 ones = f32x4{1.f, 1.f, 1.f, 1.f};
    f32x4 f_in = ones, f_out = ones, pending = ones, whole = ones;
    auto fetch_f = [&](int j) __attribute__((always_inline)) {
        const float* src = fac + ((long long)(b0 + j) * H + h) * 3 * DP + 4 * t;
        f_in = f_out = ones;
        if (t < DP / 4) {
            if (!is_marked(j)) {
                f_in = *reinterpret_cast<const f32x4*>(src);
                f_out = *reinterpret_cast<const f32x4*>(src + DP);
            }
            if (!OUT && vb == 0) whole *= *reinterpret_cast<const f32x4*>(src + 2 * DP);
        }
    };
    auto park_f = [&](int buf) __attribute__((always_inline)) {
        if (t < DP / 4) *reinterpret_cast<f32x4*>(sF + buf * DP + 4 * t) = pending * f_in;
        pending = f_out;
    };
    auto load_f = [&](f32x4 (&v)[4], const float* f, int td) __attribute__((always_inline)) {
#pragma unroll
        for (int rg = 0; rg < 4; ++rg) v[rg] = *reinterpret_cast<const f32x4*>(f + 32 * (td0 + td) + 8 * rg + 4 * h2);
    };
    auto scale_rows = [&](f32x16& x, const f32x4 (&v)[4]) __attribute__((always_inline)) {
#pragma unroll
        for (int rg = 0; rg < 4; ++rg)
#pragma unroll
            for (int e = 0; e < 4; ++e) x[4 * rg + e] *= v[rg][e];
    };
    auto scale_all = [&](const float* f) __attribute__((always_inline)) {
#pragma unroll
        for (int td = 0; td < TD; ++td) {
            f32x4 v[4];
            load_f(v, f, td);
            scale_rows(S[td], v);
            sched_fence();
        }
    };
    // LDS addresses of the fragment reads: a lane's base with the chunk index as an exclusive-or (a row's bytes in front of the chunk field are zeros, and
    // the swizzle of a row repeats every 16 rows)
    const int tr = 4 * h2 + (c16 >> 2), tc = 16 * ((l >> 4) & 1) + 4 * (l & 3);   // TileImg::columns' row and column at (0, 0)
    const int q_lane = L::Q0 + c32 * QI::ROW + 8 * h2 + (QI::swz(c32) << 4);                                  // B operand of S^T q^T, chunk 0
    const int t0_lane = L::K0 + tr * QI::ROW + (((tc >> 3) ^ QI::swz(tr)) << 4) + (tc & 7) * 2;               // transposing read of k^, channels 0 ..
    const int t1_lane = L::K0 + (tr + 8) * QI::ROW + (((tc >> 3) ^ QI::swz(tr + 8)) << 4) + (tc & 7) * 2;
    const int s_lane = c16 * QI::ROW + ((q4 ^ QI::swz(c16)) << 4);                                            // score fragments, relative to an image
    load_marks(0);
    fetch_f(0);
    if (OUT) {
        for (int i = t; i < 64 * L::PP / 8; i += NWT * 64) st16(sP + i * 8, zero16());   // (tiles above the diagonal stay zero)
        dma_q(0, 0);
    }
    dma_kv(0, 0);
    park_f(0);
    for (int j = 0; j < nb; ++j) {
        const int row0 = r_first + BLK * j, n = min(BLK, rows_all - BLK * j);
        const float* f = sF + (j & 1) * DP;
        const bool more = j + 1 < nb;
        const bool exact = is_marked(j);
        if (((j + 1) & 63) == 0) load_marks(j + 1);
        if (exact) {   // (workgroup-uniform) token by token: decays from alpha, q, k, v as they lie in proj
            barrier();
            scale_all(f);
            for (int i = 0; i < n; ++i) {
                const bf16_t* p = proj + (long long)(row0 + i) * s.ldp;
                const float* a = alpha + ((long long)(row0 + i) * H + h) * DP;
                const float v = mine ? ldf(p + s.v_off + h * s.dvp + vcol + c32) : 0.f;
                float o = 0.f;
#pragma unroll
                for (int td = 0; td < TD; ++td)
#pragma unroll
                    for (int r = 0; r < 16; ++r) {
                        const int d = 32 * (td0 + td) + acc_row(r, l);
                        S[td][r] = a[d] * S[td][r] + ldf(p + s.k_off + h * DP + d) * v;
                        if (OUT) o += S[td][r] * ldf(p + s.q_off + h * DP + d);
                        if ((r & 3) == 3) sched_fence();   // (four channels' operands at a time: the registers are the state's)
                    }
                if (OUT) {
                    o += shfl_xor(o, 32);
                    if (DS == 2) {   // (the halves' sums meet in LDS, alternating places)
                        float* sO = reinterpret_cast<float*>(smem + L::O0) + (i & 1) * NWT * 64;
                        if (ds == 1) sO[ws * 64 + l] = o;
                        barrier();
                        if (ds == 0) o += sO[ws * 64 + l];
                    }
                    if (mine && h2 == 0 && ds == 0) stf(out + ((long long)(row0 + i) * H + h) * s.dvp + vcol + c32, o);
                }
            }
            wait_vm<0>();
            barrier();
            if (more) {
                fetch_f(j + 1);
                if (OUT) dma_q(j + 1, (j + 1) & 1);
                dma_kv(j + 1, (j + 1) & 1);
                park_f((j + 1) & 1);
            }
            continue;
        }
        f32x16 o[2];
        if (OUT) {
            wait_vm<Q_PIECES + V_PIECES>();   // q^ has landed (k^ and v, requested after it, may be in flight)
            barrier();
            if (more) dma_q(j + 1, (j + 1) & 1);
            o[0] = zero_acc();
            o[1] = zero_acc();
            int ql = q_lane + (j & 1) * L::QB;
            hold(ql);
            s16x8 qf[2][4];   // [buffer][16-channel half, token half]: the next 32 channels are requested in front of this step's products
            auto load_q = [&](int td, s16x8 (&x)[4]) __attribute__((always_inline)) {
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int ch = 4 * (td0 + td) + 2 * (i >> 1);
                    const s16x4 x0 = *reinterpret_cast<const s16x4*>(smem + (ql ^ (ch << 4)) + 32 * (i & 1) * QI::ROW);
                    const s16x4 x1 = *reinterpret_cast<const s16x4*>(smem + (ql ^ ((ch + 1) << 4)) + 32 * (i & 1) * QI::ROW);
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        x[i][e] = x0[e];
                        x[i][4 + e] = x1[e];
                    }
                }
            };
            f32x4 fv[4];
            load_f(fv, f, 0);
            load_q(0, qf[0]);
#pragma unroll
            for (int td = 0; td < TD; ++td) {
                if (td + 1 < TD) load_q(td + 1, qf[(td + 1) & 1]);
                sched_fence();
                scale_rows(S[td], fv);
                if (td + 1 < TD) load_f(fv, f, td + 1);
#pragma unroll
                for (int u = 0; u < 2; ++u) {
                    const s16x8 hi = pack_frag(S[td], u);
                    f32x16 rest;
#pragma unroll
                    for (int e = 0; e < 8; ++e) rest[8 * u + e] = S[td][8 * u + e] - bf2f(bf16_t(hi[e]));
                    const s16x8 lo = pack_frag(rest, u);
#pragma unroll
                    for (int tt = 0; tt < 2; ++tt) {
                        o[tt] = mfma32(hi, qf[td & 1][2 * u + tt], o[tt]);
                        o[tt] = mfma32(lo, qf[td & 1][2 * u + tt], o[tt]);
                    }
                }
                sched_fence();
            }
            if (DS == 2) {   // the other half's partial sums of this wave's tokens, and its own of the other's
                f32x4* give = reinterpret_cast<f32x4*>(smem + L::O0 + w * 4096) + l;
#pragma unroll
                for (int rg = 0; rg < 4; ++rg) {
                    f32x4 v;
#pragma unroll
                    for (int e = 0; e < 4; ++e) v[e] = ds ? o[0][4 * rg + e] : o[1][4 * rg + e];
                    give[64 * rg] = v;
                }
#pragma unroll
                for (int r = 0; r < 16; ++r) o[0][r] = ds ? o[1][r] : o[0][r];
            }
        }
        if (OUT) {   // k^ has landed (v and the next q^ may be in flight)
            if (more)
                wait_vm<V_PIECES + Q_PIECES>();
            else
                wait_vm<V_PIECES>();
        } else {
            wait_vm<0>();
        }
        barrier();
        if (!OUT && more) dma_kv(j + 1, (j + 1) & 1);
        if (OUT && DS == 2) {
            const f32x4* take = reinterpret_cast<const f32x4*>(smem + L::O0 + (ws + (1 - ds) * NW) * 4096) + l;
#pragma unroll
            for (int rg = 0; rg < 4; ++rg) {
                const f32x4 v = take[64 * rg];
#pragma unroll
                for (int e = 0; e < 4; ++e) o[0][4 * rg + e] += v[e];
            }
        }
        if (OUT) {   // scores: 16 x 16 tiles (a, b) of the lower triangle, rows = keys 4 q4 + r, columns = queries
            for (int x = w; x < 10; x += NWT) {
                const int a = x < 1 ? 0 : x < 3 ? 1 : x < 6 ? 2 : 3, kb = x - a * (a + 1) / 2;
                f32x4 sc[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
                int sl = s_lane;
                hold(sl);
                const int qr = 16 * a + c16;
#pragma unroll
                for (int kk = 0; kk < DP / 32; ++kk) {
                    const s16x8 ka = *reinterpret_cast<const s16x8*>(smem + L::K0 + 16 * kb * QI::ROW + (sl ^ (kk << 6)));
                    const s16x8 qb = *reinterpret_cast<const s16x8*>(smem + L::Q0 + (j & 1) * L::QB + 16 * a * QI::ROW + (sl ^ (kk << 6)));
                    sc[kk & 1] = mfma16(ka, qb, sc[kk & 1]);
                }
                float p[4];
#pragma unroll
                for (int r = 0; r < 4; ++r) p[r] = a == kb && 4 * q4 + r > c16 ? 0.f : sc[0][r] + sc[1][r];
                *reinterpret_cast<u32x2*>(sP + qr * L::PP + 16 * kb + 4 * q4) = u32x2{pack2bf(p[0], p[1]), pack2bf(p[2], p[3])};
            }
            if (more)
                wait_vm<Q_PIECES>();   // v has landed
            else
                wait_vm<0>();
            barrier();   // scores complete
        }
        const char* sV = smem + L::V0 + (j & 1) * L::V_STEP;
        if (more) fetch_f(j + 1);
        s16x8 vf[4];
#pragma unroll
        for (int jb = 0; jb < 4; ++jb) vf[jb] = VI::columns(sV, 16 * jb, 32 * ws, l);
        if (OUT) {
#pragma unroll
            for (int i = 0; i < OT; ++i) {
                const int tt = DS == 2 ? ds : i;
#pragma unroll
                for (int jb = 0; jb < 4; ++jb) {
                    if (jb >= 2 && tt == 0) break;   // (the first half of the tokens sees the first half of the keys)
                    const bf16_t* src = sP + (32 * tt + c32) * L::PP + 16 * jb + 4 * h2;
                    const s16x4 x0 = *reinterpret_cast<const s16x4*>(src), x1 = *reinterpret_cast<const s16x4*>(src + 8);
                    s16x8 pf;
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        pf[e] = x0[e];
                        pf[4 + e] = x1[e];
                    }
                    o[i] = mfma32(vf[jb], pf, o[i]);
                }
                if (mine && 32 * tt + c32 < n) {
                    bf16_t* dst = out + ((long long)(row0 + 32 * tt + c32) * H + h) * s.dvp + vcol + 4 * h2;
#pragma unroll
                    for (int rg = 0; rg < 4; ++rg)
                        *reinterpret_cast<u32x2*>(dst + 8 * rg) =
                            u32x2{pack2bf(o[i][4 * rg], o[i][4 * rg + 1]), pack2bf(o[i][4 * rg + 2], o[i][4 * rg + 3])};
                }
            }
        }
        if (!OUT) scale_all(f);
        int t0 = t0_lane + (j & 1) * L::K_STEP, t1 = t1_lane + (j & 1) * L::K_STEP;
        hold(t0);
        hold(t1);
        s16x8 kf[2][4];
        auto load_k = [&](int td, s16x8 (&x)[4]) __attribute__((always_inline)) {
#pragma unroll
            for (int jb = 0; jb < 4; ++jb) {
                const s16x4 x0 = ds_read_tr16(reinterpret_cast<const bf16_t*>(smem + (t0 ^ ((td0 + td) << 6)) + 16 * jb * QI::ROW));
                const s16x4 x1 = ds_read_tr16(reinterpret_cast<const bf16_t*>(smem + (t1 ^ ((td0 + td) << 6)) + 16 * jb * QI::ROW));
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    x[jb][e] = x0[e];
                    x[jb][4 + e] = x1[e];
                }
            }
        };
        load_k(0, kf[0]);
#pragma unroll
        for (int td = 0; td < TD; ++td) {
            if (td + 1 < TD) load_k(td + 1, kf[(td + 1) & 1]);
            sched_fence();
#pragma unroll
            for (int jb = 0; jb < 4; ++jb) S[td] = mfma32(kf[td & 1][jb], vf[jb], S[td]);
            sched_fence();
        }
        if (more) park_f((j + 1) & 1);
        if (OUT) barrier();   // every wave is done with k^ and v (OUT = false: the next block's first barrier says so)
        if (OUT && more) dma_kv(j + 1, 0);
    }
    if (!OUT || last) {   // what the last block left to the next one
        f_in = ones;
        park_f(nb & 1);
        barrier();
        scale_all(sF + (nb & 1) * DP);
    }
    if (!OUT && t < DP / 4 && vb == 0) *reinterpret_cast<f32x4*>(decays + ((long long)(c + 1) * H + h) * DP + 4 * t) = whole;
    if (!mine || (OUT && !last)) return;
    float* dst = OUT ? slot_state : states + ((long long)(c + 1) * H + h) * head_state + vcol + c32;
#pragma unroll
    for (int i = 0; i < TD; ++i)
#pragma unroll
        for (int r = 0; r < 16; ++r) dst[(long long)(32 * (td0 + i) + acc_row(r, l)) * s.dvp] = S[i][r];
}

// first states of the chunks: states[c] and decays[c] hold chunk c - 1's state from zero and decay; on return states[c] is the state in front of chunk c.  A thread: four columns of one
// channel, all chunks of a sequence.
__global__ __launch_bounds__(256) void linear_scan_kernel(Lin s, const int32_t* blocks, const int32_t* chunks, const int32_t* seqs, const float* decays, float* states,
                                                          const float* cache, const int32_t* slot, const int32_t* pos) {
    const int i = blockIdx.x * 256 + threadIdx.x, h = blockIdx.y, c0 = seqs[2 * blockIdx.z], nc = seqs[2 * blockIdx.z + 1];
    const long long head_state = s.dp * s.dvp, H = s.H;
    if (nc < 2 || 4ll * i >= head_state) return;
    const int d = int(4ll * i / s.dvp), r0 = blocks[2 * chunks[4 * c0]];
    f32x4 x = f32x4{0.f, 0.f, 0.f, 0.f};
    if (pos[r0] > 0) x = *reinterpret_cast<const f32x4*>(cache + ((long long)slot[r0] * H + h) * head_state + 4 * i);
    float* at = states + ((long long)c0 * H + h) * head_state + 4 * i;
    *reinterpret_cast<f32x4*>(at) = x;
    constexpr int AHEAD = 4;
    const long long step = H * head_state;
    for (int c = 1; c < nc; c += AHEAD) {
        f32x4 own[AHEAD];
        float a[AHEAD];
#pragma unroll
        for (int u = 0; u < AHEAD; ++u) {
            const int k = min(c + u, nc - 1);
            own[u] = *reinterpret_cast<const f32x4*>(at + k * step);
            a[u] = decays[((long long)(c0 + k) * H + h) * s.dp + d];
        }
#pragma unroll
        for (int u = 0; u < AHEAD; ++u) {
            if (c + u >= nc) break;
#pragma unroll
            for (int e = 0; e < 4; ++e) x[e] = a[u] * x[e] + own[u][e];
            *reinterpret_cast<f32x4*>(at + (c + u) * step) = x;
        }
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
    float *fac, *alpha, *states, *decays;
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
    z.decays = reinterpret_cast<float*>(take(4 * n_chunks * s.H * s.dp));
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
    using L = ChunkSmem<DP, NW, true>;
    const Lin& s = a.s;
    const int64_t nvb = (s.dvp + L::VB - 1) / L::VB;
    const dim3 grid(unsigned(8 * nvb * ((s.H * a.n_chunks + 7) / 8))), block(L::WAVES * 64);
    if (a.n_chunks > a.n_seq) {
        ARIA_LAUNCH((linear_chunk_kernel<DP, NW, false>), grid, block, size_t(ChunkSmem<DP, NW, false>::BYTES), a.stream, (const bf16_t*)a.proj, s, a.blocks,
                    a.chunks, (const float*)a.z.fac, (const int32_t*)a.z.marked, (const float*)a.z.alpha, a.z.states, a.z.decays, a.state, a.slot, a.pos, a.out,
                    int(a.n_chunks));
        const int64_t n4 = s.dp * s.dvp / 4;
        ARIA_LAUNCH(linear_scan_kernel, dim3(unsigned((n4 + 255) / 256), unsigned(s.H), unsigned(a.n_seq)), dim3(256), 0, a.stream, s, a.blocks, a.chunks,
                    a.seqs, (const float*)a.z.decays, a.z.states, (const float*)a.state, a.slot, a.pos);
    }
    ARIA_LAUNCH((linear_chunk_kernel<DP, NW, true>), grid, block, size_t(L::BYTES), a.stream, (const bf16_t*)a.proj, s, a.blocks, a.chunks, (const float*)a.z.fac,
                (const int32_t*)a.z.marked, (const float*)a.z.alpha, a.z.states, a.z.decays, a.state, a.slot, a.pos, a.out, int(a.n_chunks));
    return aria_check_launch();
}
template <int DP>
int run_chunks(const ChunkArgs& a) {
    const size_t lds = size_t((PREP / (DP / 2) + 1) * DP + 8 + BLK * a.s.rank) * 4;
    if (lds > 160 * 1024) return ARIA_ERR_UNSUPPORTED;
    ARIA_LAUNCH((linear_prepare_kernel<DP>), dim3(unsigned(a.n_blocks), unsigned(a.s.H)), dim3(PREP), lds, a.stream, a.proj, a.s, a.blocks, a.z.fac, a.z.marked,
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
