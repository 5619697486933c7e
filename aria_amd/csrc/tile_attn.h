// Decode attention on the matrix pipe (bf16): cache rows that serve many query heads -- latent rows shared by all heads, or the [key | value] rows of one
// key / value head and its group of query heads -- are a matrix product's operand streamed from HBM, the heads its rows.
#pragma once
#include "elem.h"

namespace ad {

struct TileAttn {
    const bf16_t* q;                     // query of (token, head) at q + token q_tok + head q_head, kc columns
    long long q_tok;
    int q_head;
    const bf16_t* cache;                 // row r of (slot, kv head g) at cache + slot slot_stride + g group_stride + r cw
    long long slot_stride, group_stride;
    int cw, kc, vo, R;                   // a cache row; its columns [0, kc) meet the query, [vo, vo + R) are summed
    int H, Hg;                           // query heads, query heads per kv head
    int window;                          // 0: a token sees rows 0 .. pos; else rows 0 .. pos % window
    float scale;
};

// One workgroup of 8 waves: one token, NG groups of 16 heads, a contiguous range of 64-row cache tiles.  Tiles arrive by LDS-DMA, double-buffered,
// chunk slot = chunk ^ tile_swz(row).  Per tile: wave w scores rows 16 (w & 3) .. against head group w >> 2 (NG = 1: against the half of the reduction
// w >> 2; cache rows are k-contiguous B fragments as they lie) and parks the scores in LDS; wave w then owns the softmax of 2 NG heads, a lane per
// row (DPP reductions, running maximum and sum in registers), and publishes probabilities (bf16) and rescale factors; last, wave w accumulates DTW
// 16-column slices of the output over all 64 rows (V fragments by transposing reads of the same tile).  Softmax in the log2 domain, fp32.
// XOR of a chunk index inside its group of 8: a row is an odd multiple of 32 banks (or an even one) behind its neighbour, so the 16 rows of a score
// fragment (8 of either parity) need 8 different values, and the 16 (row, 32-byte) pairs of a transposing read need all four upper-bit values twice
__device__ __forceinline__ int tile_swz(int row) { return ((((row >> 1) ^ (row >> 3)) & 3) << 1) | ((row >> 3) & 1); }
namespace {
template <int NG, int DTW, int KTM>
__global__ __launch_bounds__(512) void tile_attn_kernel(TileAttn s, const int32_t* slot, const int32_t* pos, float* part_o, float* part_ml, int splits) {
    ARIA_DYN_SMEM(smem);
    constexpr int PP = 72, SPI = 66;   // pitches of the probability tile (bf16) and of the score tile (fp32)
    constexpr int NP = NG == 1 ? 2 : 1;   // partial score tiles (halves of the reduction)
    constexpr int KW = (KTM + NP - 1) / NP, HW = 2 * NG;
    const int t = threadIdx.x, l = t & 63, w = first_lane(t >> 6), q4 = l >> 4, c16 = l & 15;
    const int CPR = s.cw >> 3, KT = s.kc >> 5, tile_bytes = 64 * s.cw * 2;
    float* sS = reinterpret_cast<float*>(smem + 2 * tile_bytes);                 // [NP][NG * 16][SPI]
    bf16_t* sP = reinterpret_cast<bf16_t*>(sS + NP * NG * 16 * SPI);             // [NG * 16][PP]
    float* sA = reinterpret_cast<float*>(sP + NG * 16 * PP);                     // [NG * 16]
    const int sp = blockIdx.x, sets = (s.Hg + 16 * NG - 1) / (16 * NG), kvh = int(blockIdx.y) / sets, tok = blockIdx.z;
    const int n_keys = (s.window ? pos[tok] % s.window : pos[tok]) + 1, ntiles = (n_keys + 63) / 64, per = (ntiles + splits - 1) / splits;
    const int it0 = sp * per, it1 = min(ntiles, it0 + per);
    const int head0 = kvh * s.Hg + (int(blockIdx.y) % sets) * NG * 16, head_end = (kvh + 1) * s.Hg;
    float* ml = part_ml + ((long long)tok * splits + sp) * s.H * 2;
    if (it0 >= it1) {   // nothing to see for this split
        if (t < NG * 16 && head0 + t < head_end) {
            ml[2 * (head0 + t)] = -INFINITY;
            ml[2 * (head0 + t) + 1] = 0.f;
        }
        return;
    }
    const bf16_t* base = s.cache + slot[tok] * s.slot_stride + kvh * s.group_stride;
    // this lane's chunk of the wave's first DMA piece, and the step to its next one (8 pieces of 64 chunks further on)
    const int row_i = (w * 64 + l) / CPR, slot_i = (w * 64 + l) % CPR, dr_ = 512 / CPR, ds_ = 512 % CPR;
    auto dma = [&](int tile, char* dst) __attribute__((always_inline)) {
        int row = row_i, sl = slot_i;
        for (int pc = w; pc < CPR; pc += 8) {
            const int ch = sl ^ tile_swz(row);
            glds16_raw(base + (long long)min(tile * 64 + row, n_keys - 1) * s.cw + ch * 8, dst + pc * 1024);
            row += dr_;
            sl += ds_;
            if (sl >= CPR) {
                sl -= CPR;
                row += 1;
            }
        }
    };
    dma(it0, smem);
    const int g = NG == 1 ? 0 : w >> 2, k_first = NG == 1 ? (w >> 2) * KW : 0, krow = 16 * (w & 3) + c16;
    s16x8 qf[KW];
#pragma unroll
    for (int kk = 0; kk < KW; ++kk) {
        u32x4 v = zero16();
        const int head = head0 + g * 16 + c16;
        if (head < head_end && k_first + kk < KT) v = ld16(s.q + tok * s.q_tok + (long long)head * s.q_head + (k_first + kk) * 32 + q4 * 8);
        qf[kk] = __builtin_bit_cast(s16x8, v);
    }
    f32x4 o[NG][DTW];
#pragma unroll
    for (int gg = 0; gg < NG; ++gg)
#pragma unroll
        for (int i = 0; i < DTW; ++i) o[gg][i] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m[HW], lsum[HW];
#pragma unroll
    for (int j = 0; j < HW; ++j) {
        m[j] = -INFINITY;
        lsum[j] = 0.f;
    }
#pragma unroll
    for (int kk = 0; kk < KW; ++kk) settle(qf[kk]);
    const float scale2 = s.scale * 1.4426950408889634f;
    for (int it = it0; it < it1; ++it) {
        const char* cur = smem + ((it - it0) & 1) * tile_bytes;
        wait_vm<0>();
        sync();   // tile `it` is complete; every wave is done with the other buffer and the probabilities
        if (it + 1 < it1) dma(it + 1, smem + ((it - it0 + 1) & 1) * tile_bytes);
        {   // scores: C rows = heads 4 q4 + r of group g, columns = cache rows
            // (no branch on the row's width: blocks past it read the last chunk against zero query fragments; the next group's fragments are
            // requested in front of this group's multiply-adds)
            constexpr int GQ = KW % 3 == 0 ? 3 : 5;
            f32x4 sc[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
            const char* kbase = cur + krow * CPR * 16;
            const int fx = tile_swz(krow);
            s16x8 kf[2][GQ];
            auto fetch = [&](int kk, s16x8& f) __attribute__((always_inline)) {
                f = *reinterpret_cast<const s16x8*>(kbase + ((min((k_first + kk) * 4 + q4, CPR - 1) ^ fx) << 4));
            };
#pragma unroll
            for (int u = 0; u < GQ; ++u) fetch(u, kf[0][u]);
#pragma unroll
            for (int k0 = 0; k0 < KW; k0 += GQ) {
                if (k0 + GQ < KW) {
#pragma unroll
                    for (int u = 0; u < GQ; ++u) fetch(k0 + GQ + u, kf[(k0 / GQ + 1) & 1][u]);
                }
                sched_fence();
#pragma unroll
                for (int u = 0; u < GQ; ++u) sc[u & 1] = mfma16(qf[k0 + u], kf[(k0 / GQ) & 1][u], sc[u & 1]);
                sched_fence();
            }
            float* dst = sS + ((NG == 1 ? w >> 2 : 0) * NG * 16 + g * 16 + 4 * q4) * SPI + krow;
#pragma unroll
            for (int r = 0; r < 4; ++r) dst[r * SPI] = sc[0][r] + sc[1][r];
        }
        sync();
        // softmax: lane = row of the tile
        const bool dead = it * 64 + l >= n_keys;
        float x[HW], mx[HW];
#pragma unroll
        for (int j = 0; j < HW; ++j) {
            x[j] = sS[(w * HW + j) * SPI + l];
            if (NP == 2) x[j] += sS[(NG * 16 + w * HW + j) * SPI + l];
        }
#pragma unroll
        for (int j = 0; j < HW; ++j) mx[j] = x[j] = dead ? -INFINITY : x[j] * scale2;
        wave_max_bcast_n<HW>(mx);
#pragma unroll
        for (int j = 0; j < HW; ++j) {
            const float mn = fmaxf(m[j], mx[j]);   // finite: a tile holds at least one visible row
            const float alpha = exp2_fast(m[j] - mn), p = exp2_fast(x[j] - mn);
            m[j] = mn;
            lsum[j] = lsum[j] * alpha + p;
            sP[(w * HW + j) * PP + l] = f2bf(p);
            if (l == 0) sA[w * HW + j] = alpha;
        }
        sync();
        // output: A = probabilities (heads x 32 rows), B = the tile's columns
#pragma unroll
        for (int gg = 0; gg < NG; ++gg) {
            const f32x4 al = *reinterpret_cast<const f32x4*>(sA + gg * 16 + 4 * q4);
#pragma unroll
            for (int i = 0; i < DTW; ++i)
#pragma unroll
                for (int r = 0; r < 4; ++r) o[gg][i][r] *= al[r];
        }
        s16x8 pf[2][NG], vf[2][DTW];
        auto fetch_v = [&](int kk) __attribute__((always_inline)) {
#pragma unroll
            for (int gg = 0; gg < NG; ++gg) pf[kk][gg] = *reinterpret_cast<const s16x8*>(sP + (gg * 16 + c16) * PP + kk * 32 + q4 * 8);
            const int vr = kk * 32 + q4 * 8 + (c16 >> 2);
#pragma unroll
            for (int i = 0; i < DTW; ++i) {
                const int d0 = min(s.vo + (w * DTW + i) * 16, s.cw - 16);   // (slices past the row: any columns, their results are dropped)
                const int col = d0 + 4 * (c16 & 3), ch = col >> 3, within = (col & 7) * 2;
                const s16x4 a0 = ds_read_tr16(reinterpret_cast<const bf16_t*>(cur + vr * CPR * 16 + ((ch ^ tile_swz(vr)) << 4) + within));
                const s16x4 a1 = ds_read_tr16(reinterpret_cast<const bf16_t*>(cur + (vr + 4) * CPR * 16 + ((ch ^ tile_swz(vr + 4)) << 4) + within));
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    vf[kk][i][e] = a0[e];
                    vf[kk][i][4 + e] = a1[e];
                }
            }
        };
        fetch_v(0);
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
            if (kk == 0) fetch_v(1);
            sched_fence();
#pragma unroll
            for (int i = 0; i < DTW; ++i)
#pragma unroll
                for (int gg = 0; gg < NG; ++gg) o[gg][i] = mfma16(pf[kk][gg], vf[kk][i], o[gg][i]);
            sched_fence();
        }
    }
#pragma unroll
    for (int j = 0; j < HW; ++j) {
        const float v = wave_sum_bcast(lsum[j]);
        const int head = head0 + w * HW + j;
        if (l == 0 && head < head_end) {
            ml[2 * head] = m[j];
            ml[2 * head + 1] = v;
        }
    }
#pragma unroll
    for (int gg = 0; gg < NG; ++gg)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int head = head0 + gg * 16 + 4 * q4 + r;
            if (head >= head_end) continue;
            float* po = part_o + (((long long)tok * splits + sp) * s.H + head) * s.R;
#pragma unroll
            for (int i = 0; i < DTW; ++i) {
                const int d = (w * DTW + i) * 16 + c16;
                if (d < s.R) po[d] = o[gg][i][r];
            }
        }
}
}  // namespace

constexpr int TILE_MAX_SPLITS = 64;
// the kernel's limits: 1, 2, 3 = the instantiation that holds the shape, 0 = none
inline int tile_attn_class(int64_t kc, int64_t R, int64_t cw) {
    if ((cw & 63) || (kc & 31) || cw > 576) return 0;
    if (R <= 128 && kc <= 192) return 1;
    if (R <= 256 && kc <= 320) return 2;
    if (R <= 512 && kc <= 576) return 3;
    return 0;
}
// one round of workgroups: as many as the 256 CUs hold at a time (a workgroup's LDS is two cache tiles), no more -- a workgroup's start and end cost
// as much as two tiles
inline int64_t tile_attn_splits(int64_t cw, int64_t H, int64_t Hg, int64_t T, int64_t max_keys) {
    const int64_t tiles = (max_keys + 63) / 64, sets = (H / Hg) * (Hg <= 16 ? 1 : (Hg + 31) / 32);
    const int64_t per_cu = (2 * 64 * cw * 2 + 16 * 1024) * 2 <= 160 * 1024 ? 2 : 1;
    int64_t n = 256 * per_cu / (T * sets);
    n = n < tiles ? n : tiles;
    n = n < TILE_MAX_SPLITS ? n : TILE_MAX_SPLITS;
    return n < 1 ? 1 : n;
}
// part_o fp32 [T, splits, H, R] unnormalised outputs, part_ml fp32 [T, splits, H, 2] (running maximum in log2 units, sum)
static inline int launch_tile_attn(const TileAttn& s, const int32_t* slot, const int32_t* pos, float* part_o, float* part_ml, int64_t T, int64_t splits, void* stream) {
    const int cls = tile_attn_class(s.kc, s.R, s.cw);
    const int NG = s.Hg <= 16 ? 1 : 2;
    const dim3 grid(unsigned(splits), unsigned((s.H / s.Hg) * ((s.Hg + 16 * NG - 1) / (16 * NG))), static_cast<unsigned>(T)), block(512);
    const size_t lds = size_t(2) * 64 * s.cw * 2 + size_t(32) * 66 * 4 + size_t(NG) * 16 * (72 * 2 + 4);
    if (!cls || T > 65535 || splits > TILE_MAX_SPLITS || lds > 160 * 1024) return ARIA_ERR_UNSUPPORTED;
#define ARIA_TILE_ATTN(G, D, K) ARIA_LAUNCH((tile_attn_kernel<G, D, K>), grid, block, lds, stream, s, slot, pos, part_o, part_ml, int(splits))
    if (NG == 1) {
        if (cls == 1)
            ARIA_TILE_ATTN(1, 1, 6);
        else if (cls == 2)
            ARIA_TILE_ATTN(1, 2, 10);
        else
            ARIA_TILE_ATTN(1, 4, 18);
    } else {
        if (cls == 1)
            ARIA_TILE_ATTN(2, 1, 6);
        else if (cls == 2)
            ARIA_TILE_ATTN(2, 2, 10);
        else
            ARIA_TILE_ATTN(2, 4, 18);
    }
#undef ARIA_TILE_ATTN
    return aria_check_launch();
}

}  // namespace ad
