// 64-row operand tiles in LDS as the attention kernels use them: images filled by LDS-DMA, their fragment reads, and the register layout of a 32 x 32
// accumulator.
#pragma once
#include "aria_device.h"

namespace ad {

__device__ __forceinline__ int acc_row(int r, int l) { return (r & 3) + 8 * (r >> 2) + 4 * (l >> 5); }
__device__ __forceinline__ f32x16 zero_acc() {
    f32x16 z;
#pragma unroll
    for (int r = 0; r < 16; ++r) z[r] = 0.f;
    return z;
}

// accumulator regs 8u..8u+7 of a 32x32 tile -> bf16 fragment (lane-local)
__device__ __forceinline__ s16x8 pack_frag(const f32x16& p, int u) {
    u32x4 v;
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = pack2bf(p[8 * u + 2 * j], p[8 * u + 2 * j + 1]);
    return __builtin_bit_cast(s16x8, v);
}

__device__ __forceinline__ int swz3(int row) { return ((row & 3) << 2) | ((row >> 2) & 3); }

// A tile of 64 rows x COLS columns (a multiple of 64).  A row is CPR 16-byte chunks; image slot s of row r holds source chunk s ^ swz(r).  swz spreads
// the rows of a fragment read over the banks: 16-chunk multiples take the 4-bit swizzle of the 128-column image, the others 3 bits (row >> 1 where
// consecutive rows already lie 32 banks apart).
template <int COLS>
struct TileImg {
    static constexpr int CPR = COLS / 8, ROW = COLS * 2, BYTES = 64 * ROW, PIECES = CPR / 8;   // 1 KiB pieces per wave
    static_assert(COLS % 64 == 0, "8 waves deal whole pieces");
    static __device__ __forceinline__ int swz(int row) { return CPR % 16 == 0 ? swz3(row) : (CPR % 16 == 8 && CPR > 8) ? (row >> 1) & 7 : row & 7; }
    int row[PIECES], col[PIECES];   // this lane's source row inside the tile and source column, per piece
    __device__ __forceinline__ void init(int w, int l) {
#pragma unroll
        for (int i = 0; i < PIECES; ++i) {
            const int c = (w + 8 * i) * 64 + l;
            row[i] = c / CPR;
            col[i] = ((c % CPR) ^ swz(row[i])) * 8;
        }
    }
    __device__ __forceinline__ void dma(const bf16_t* base, long long ld, int row0, int row_last, char* s, int w) const {
#pragma unroll
        for (int i = 0; i < PIECES; ++i) glds16_raw(base + (long long)min(row0 + row[i], row_last) * ld + col[i], s + (w + 8 * i) * 1024);
    }
    static __device__ __forceinline__ s16x8 rows(const char* s, int r, int kk, int l) {
        return *reinterpret_cast<const s16x8*>(s + r * ROW + (((2 * kk + (l >> 5)) ^ swz(r)) << 4));
    }
    static __device__ __forceinline__ s16x8 columns(const char* s, int rb, int d0, int l) {   // frag_tr3's contract
        const int r = rb + 4 * (l >> 5) + ((l & 15) >> 2);
        const int c = d0 + 16 * ((l >> 4) & 1) + 4 * (l & 3);
        const int ch = c >> 3, within = (c & 7) * 2;
        const s16x4 a0 = ds_read_tr16(reinterpret_cast<const bf16_t*>(s + r * ROW + ((ch ^ swz(r)) << 4) + within));
        const s16x4 a1 = ds_read_tr16(reinterpret_cast<const bf16_t*>(s + (r + 8) * ROW + ((ch ^ swz(r + 8)) << 4) + within));
        s16x8 f;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            f[e] = a0[e];
            f[4 + e] = a1[e];
        }
        return f;
    }
};

}  // namespace ad
