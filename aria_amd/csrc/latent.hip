// Latent attention: every head's keys and values are linear images of one low-rank latent per token, so the cache holds the latent and one
// rotated key part shared by the heads (R + dr numbers a token instead of 2 H hd).
//
// Prefill expands the latents of the new tokens to per-head keys and values (a GEMM on the packed cache rows whose weight carries identity rows for
// the rotated part) and runs the flash kernel of attn.hip on unequal query / value head widths.  Decode -- and a prompt that continues on a cache --
// never expands: the query moves into latent space once (q W_uk, per head), scores are dot products with the cache rows as they lie in memory, and
// the weighted sum of latents is expanded through W_uv at the end.  A cache row is then read ONCE for 16 or 32 heads, which makes decode
// attention a matrix product with the heads as rows (v_mfma_f32_16x16x32_bf16) whose operand streams from HBM.
#include "rows.h"
#include "tile_attn.h"
#include <cstdlib>

namespace {
using namespace ad;
typedef AriaLatentShape Shape;

// column i of a cache row: RMS-normed latent | rotated key part | zeros.  src = the token's down-projection (R + dr columns), r = 1 / rms
template <class T>
__device__ __forceinline__ float latent_column(const T* src, const Shape& s, const float* cs, const float* wn, float r, int i) {
    if (i < s.R) return ldf(src + i) * r * wn[i];
    if (i >= s.R + s.dr) return 0.f;
    const int j = i - int(s.R), half = int(s.rot) >> 1;
    const float v = ldf(src + i);
    if (j < half) return v * cs[2 * j] - ldf(src + i + half) * cs[2 * j + 1];
    if (j < s.rot) return v * cs[2 * (j - half)] + ldf(src + i - half) * cs[2 * (j - half) + 1];
    return v;
}

// ---------------------------------------------------------------------------------------------- prefill: rotate q, write the cache
template <class T>
__global__ __launch_bounds__(256) void latent_rows_kernel(T* proj, Shape s, const int32_t* slot, const int32_t* pos, const float* rope,
                                                          const float* wn, T* cache, T* packed, int n_tok) {
    const int l = threadIdx.x & 63;
    const int t = (blockIdx.x * blockDim.x + threadIdx.x) >> 6;
    if (t >= n_tok) return;
    T* p = proj + (long long)t * s.ldp;
    const int ps = pos[t];
    const float* cs = rope + (long long)ps * s.rot;
    const T* src = p + s.kv_off;
    float ss = 0.f;
    for (int i = l; i < s.R; i += 64) {
        const float v = ldf(src + i);
        ss += v * v;
    }
    const float r = 1.f / sqrtf(wave_sum_bcast(ss) / float(s.R) + s.eps);
    T *row = cache + ((long long)slot[t] * s.S_cap + ps) * s.cw, *prow = packed + (long long)t * s.cw;
    for (int i = l; i < s.cw; i += 64) {
        const float v = latent_column<T>(src, s, cs, wn, r, i);
        stf(row + i, v);
        stf(prow + i, v);
    }
    const int half = int(s.rot) >> 1;
    for (int i = l; i < s.H * half; i += 64) {
        const int h = i / half, j = i % half;
        T* a = p + (long long)h * s.dq + s.dn + j;
        const float u = ldf(a), v = ldf(a + half), c = cs[2 * j], sn = cs[2 * j + 1];
        stf(a, u * c - v * sn);
        stf(a + half, v * c + u * sn);
    }
}

// ---------------------------------------------------------------------------------------------- decode: queries into latent space
// grid (H * RB + 1, token groups): workgroup (h, rb) computes 128 latent columns of head h for NB tokens -- 16 column groups of 8 x 16 slices of the
// reduction over dn, a thread's eight weight rows requested before the queries are staged -- and, at rb = 0, the head's rotated query part; the last
// workgroup of a token group writes the cache rows.
template <class T>
struct Pack8 {   // 8 elements in registers as they came from memory
    u32x4 v[sizeof(T) / 2];
    __device__ __forceinline__ void load(const T* p) {
#pragma unroll
        for (int i = 0; i < int(sizeof(T) / 2); ++i) v[i] = ld16(reinterpret_cast<const char*>(p) + 16 * i);
    }
    __device__ __forceinline__ float at(int e) const {
        if (sizeof(T) == 2) return e & 1 ? bfhi(v[0][e >> 1]) : bflo(v[0][e >> 1]);
        const uint32_t bits = v[(sizeof(T) / 4) * (e >> 2)][e & 3];   // (a bit_cast of the element itself reads element 0)
        return __builtin_bit_cast(float, bits);
    }
};
template <class T, int NB>
__global__ __launch_bounds__(256) void latent_absorb_kernel(const T* proj, Shape s, const int32_t* slot, const int32_t* pos, const float* rope,
                                                            const float* wn, const T* uk, T* cache, T* qa, int n_tok) {
    ARIA_DYN_SMEM(smem);
    float* red = reinterpret_cast<float*>(smem);   // [16][NB][128]
    float* sq = red + 16 * NB * 128;               // [NB][dn]
    const int t = threadIdx.x, l = t & 63, w = t >> 6;
    const int RB = int(s.R + 127) / 128, unit = blockIdx.x, t0 = blockIdx.y * NB;
    const int nb = min(NB, n_tok - t0), half = int(s.rot) >> 1;
    if (unit == s.H * RB) {   // cache rows: the whole workgroup on one token at a time
        for (int b = 0; b < nb; ++b) {
            const int tok = t0 + b, ps = pos[tok];
            const T* src = proj + (long long)tok * s.ldp + s.kv_off;
            float ss = 0.f;
            for (int i = t; i < s.R; i += 256) {
                const float v = ldf(src + i);
                ss += v * v;
            }
            ss = wave_sum_bcast(ss);
            sync();
            if (l == 0) red[w] = ss;
            sync();
            const float r = 1.f / sqrtf((red[0] + red[1] + red[2] + red[3]) / float(s.R) + s.eps);
            T* row = cache + ((long long)slot[tok] * s.S_cap + ps) * s.cw;
            for (int i = t; i < s.cw; i += 256) stf(row + i, latent_column<T>(src, s, rope + (long long)ps * s.rot, wn, r, i));
        }
        return;
    }
    const int h = unit / RB, r0 = (unit % RB) * 128, cg = t & 15, g = t >> 4;
    const int col = r0 + cg * 8, dn = int(s.dn);
    const T* wp = uk + (long long)h * dn * s.rp + (col < s.rp ? col : 0);
    float acc[NB][8];
#pragma unroll
    for (int b = 0; b < NB; ++b)
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[b][e] = 0.f;
    for (int d0 = 0; d0 < dn; d0 += 128) {
        Pack8<T> wv[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) wv[i].load(wp + (long long)min(d0 + 16 * i + g, dn - 1) * s.rp);
        if (d0 == 0) {
            for (int i = t; i < NB * dn; i += 256) {
                const int b = i / dn;
                sq[i] = ldf(proj + (long long)(t0 + min(b, nb - 1)) * s.ldp + (long long)h * s.dq + i % dn);
            }
            sync();
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const int d = d0 + 16 * i + g;
#pragma unroll
            for (int b = 0; b < NB; ++b) {
                const float q = d < dn ? sq[b * dn + d] : 0.f;
#pragma unroll
                for (int e = 0; e < 8; ++e) acc[b][e] += q * wv[i].at(e);
            }
        }
    }
#pragma unroll
    for (int b = 0; b < NB; ++b)
#pragma unroll
        for (int e = 0; e < 8; ++e) red[(g * NB + b) * 128 + cg * 8 + e] = acc[b][e];
    sync();
    for (int i = t; i < nb * 128; i += 256) {
        const int b = i >> 7, c = i & 127;
        if (r0 + c >= s.R) continue;
        float v = 0.f;
#pragma unroll
        for (int j = 0; j < 16; ++j) v += red[(j * NB + b) * 128 + c];
        stf(qa + ((long long)(t0 + b) * s.H + h) * s.cw + r0 + c, v);
    }
    if (r0 == 0) {   // the head's rotated part, zeros behind it
        const int extra = int(s.cw - s.R);
        for (int i = t; i < nb * extra; i += 256) {
            const int b = i / extra, j = i % extra, tok = t0 + b;
            const T* a = proj + (long long)tok * s.ldp + (long long)h * s.dq + s.dn + j;
            const float* cs = rope + (long long)pos[tok] * s.rot;
            float v = 0.f;
            if (j < s.dr) {
                v = ldf(a);
                if (j < half)
                    v = v * cs[2 * j] - ldf(a + half) * cs[2 * j + 1];
                else if (j < s.rot)
                    v = v * cs[2 * (j - half)] + ldf(a - half) * cs[2 * (j - half) + 1];
            }
            stf(qa + ((long long)tok * s.H + h) * s.cw + s.R + j, v);
        }
    }
}

// ---------------------------------------------------------------------------------------------- decode attention, any size (fp32 or bf16)
// One workgroup per (head, token), a thread per cache row of a 256-row tile, then a thread per latent column.
constexpr int ANY_COLS = 8;   // latent columns per thread: R <= 2048
template <class T>
__global__ __launch_bounds__(256) void latent_attn_any_kernel(const T* qa, const T* cache, Shape s, const int32_t* slot, const int32_t* pos,
                                                              float* part_o, float* part_ml) {
    ARIA_DYN_SMEM(smem);
    float* sq = reinterpret_cast<float*>(smem);   // [cw]
    float* sp = sq + s.cw;                        // [256]
    float* sr = sp + 256;                         // [8]
    const int t = threadIdx.x, l = t & 63, w = t >> 6, h = blockIdx.x, tok = blockIdx.y;
    const int n_keys = pos[tok] + 1, width = int(s.R + s.dr);
    const T* base = cache + (long long)slot[tok] * s.S_cap * s.cw;
    const T* q = qa + ((long long)tok * s.H + h) * s.cw;
    for (int i = t; i < s.cw; i += 256) sq[i] = ldf(q + i);
    float acc[ANY_COLS], m = -INFINITY, lsum = 0.f;
#pragma unroll
    for (int j = 0; j < ANY_COLS; ++j) acc[j] = 0.f;
    const float scale2 = s.scale * 1.4426950408889634f;
    sync();
    for (int k0 = 0; k0 < n_keys; k0 += 256) {
        float x = -INFINITY;
        if (k0 + t < n_keys) {
            const T* row = base + (long long)(k0 + t) * s.cw;
            float d = 0.f;
            for (int c = 0; c < width; c += 8) {   // (the row and the query are zero behind `width`)
                float v[8];
                ld8(row + c, v);
#pragma unroll
                for (int e = 0; e < 8; ++e) d += v[e] * sq[c + e];
            }
            x = d * scale2;
        }
        float mx = wave_max(x);
        if (l == 0) sr[w] = mx;
        sync();
        const float mn = fmaxf(m, fmaxf(fmaxf(sr[0], sr[1]), fmaxf(sr[2], sr[3])));
        const float p = exp2f(x - mn), alpha = exp2f(m - mn);
        sp[t] = p;
        const float ws = wave_sum(p);
        if (l == 0) sr[4 + w] = ws;
        sync();
        m = mn;
        lsum = lsum * alpha + (sr[4] + sr[5] + sr[6] + sr[7]);
        const int n = min(256, n_keys - k0);
#pragma unroll
        for (int j = 0; j < ANY_COLS; ++j) {
            const int r = t + 256 * j;
            if (r < s.R) {
                float a = acc[j] * alpha;
                const T* colp = base + (long long)k0 * s.cw + r;
                for (int i = 0; i < n; ++i) a += sp[i] * ldf(colp + (long long)i * s.cw);
                acc[j] = a;
            }
        }
        sync();
    }
    float* po = part_o + ((long long)tok * s.H + h) * s.R;
#pragma unroll
    for (int j = 0; j < ANY_COLS; ++j)
        if (t + 256 * j < s.R) po[t + 256 * j] = acc[j];
    if (t == 0) {
        part_ml[((long long)tok * s.H + h) * 2] = m;
        part_ml[((long long)tok * s.H + h) * 2 + 1] = lsum;
    }
}

// ---------------------------------------------------------------------------------------------- decode: merge, expand, gate
constexpr int EXP_ROWS = 32;       // value columns per workgroup: 4 per wave
constexpr int MAX_SPLITS = TILE_MAX_SPLITS;
template <class T>
__global__ __launch_bounds__(512) void latent_expand_kernel(const float* part_o, const float* part_ml, Shape s, const T* proj, const T* uv, T* out,
                                                            int splits) {
    ARIA_DYN_SMEM(smem);
    float* lat = reinterpret_cast<float*>(smem);   // [rp], zero behind R
    float* wt = lat + s.rp;                        // [MAX_SPLITS]
    const int t = threadIdx.x, l = t & 63, w = t >> 6, h = blockIdx.x, v0 = blockIdx.y * EXP_ROWS, tok = blockIdx.z;
    const int nch = int(s.rp) >> 3;
    // the wave's weight rows (their first 512 columns) are requested before the latent is merged
    Pack8<T> wv[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) wv[i].load(uv + ((long long)h * s.dv + min(v0 + w * 4 + i, int(s.dv) - 1)) * s.rp + min(l, nch - 1) * 8);
    const float gate_logit = ldf(proj + (long long)tok * s.ldp + s.g_off + h);
    if (w == 0) {
        float m = -INFINITY, sum = 0.f;
        if (l < splits) {
            const float* ml = part_ml + (((long long)tok * splits + l) * s.H + h) * 2;
            m = ml[0];
            sum = ml[1];
        }
        const float mx = wave_max_bcast(m);
        const float f = sum > 0.f ? exp2f(m - mx) : 0.f;
        const float tot = wave_sum_bcast(sum * f);
        if (l < splits) wt[l] = f / tot;
    }
    sync();
    for (int r = t; r < s.rp; r += 512) {
        float v = 0.f;
        if (r < s.R) {
            const float* p = part_o + (((long long)tok * splits) * s.H + h) * s.R + r;
            const long long step = s.H * s.R;
            for (int j = 0; j < splits; j += 16) {   // (a split without rows left its slab unwritten: selected away, not multiplied)
                float x[16];
#pragma unroll
                for (int u = 0; u < 16; ++u) x[u] = p[min(j + u, splits - 1) * step];
#pragma unroll
                for (int u = 0; u < 16; ++u) {
                    const float f = j + u < splits ? wt[min(j + u, splits - 1)] : 0.f;
                    v += f != 0.f ? f * x[u] : 0.f;
                }
            }
        }
        lat[r] = v;
    }
    sync();
    const float gate = sigmoid_exact(gate_logit);
    T* orow = out + ((long long)tok * s.H + h) * s.dvp;
    float acc[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[i] = 0.f;
    for (int c = l; c < nch; c += 64) {
        float lv[8];
        ld8(lat + c * 8, lv);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            if (c != l) wv[i].load(uv + ((long long)h * s.dv + min(v0 + w * 4 + i, int(s.dv) - 1)) * s.rp + c * 8);
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[i] += wv[i].at(e) * lv[e];
        }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const float v = wave_sum_bcast(acc[i]);
        const int col = v0 + w * 4 + i;
        if (l == 0 && col < s.dvp) stf(orow + col, col < s.dv ? v * gate : 0.f);
    }
}

// ---------------------------------------------------------------------------------------------- decode: epilogues of the projections (rows.h)
// the residual step of one stream element: x += post(v), and the next norm of the new x
__device__ __forceinline__ void stream_step(float v, const AriaDyT& post, const AriaDyT& next, float* x, bf16_t* h, long long at, int n) {
    const float xn = x[at] + dyt<bf16_t>(post, v, n);
    x[at] = xn;
    if (next.w) h[at] = f2bf(dyt<bf16_t>(next, xn, n));
}
enum { ROWS_BF16 = 0, ROWS_RELU2 = 1, ROWS_STREAM = 2, ROWS_F32 = 3 };
struct RowsOut {
    void* out;
    long long ldo;
    AriaDyT post, next;
    float* x;
    bf16_t* h;
};
template <int MODE>
struct LatentRows {
    static constexpr bool SUMSQ = false;
    RowsOut ro;
    float* sums = nullptr;
    __device__ __forceinline__ float operator()(float v, int tok, int n, int) const {
        const long long at = (long long)tok * ro.ldo + n;
        if (MODE == ROWS_BF16) static_cast<bf16_t*>(ro.out)[at] = f2bf(v);
        if (MODE == ROWS_RELU2) static_cast<bf16_t*>(ro.out)[at] = f2bf(relu_squared(v));
        if (MODE == ROWS_F32) static_cast<float*>(ro.out)[at] = v;
        if (MODE == ROWS_STREAM) stream_step(v, ro.post, ro.next, ro.x, ro.h, at, n);
        return 0.f;
    }
};

// routed up-projection of one (token, slot): act = silu(gate . h) * (up . h); the routing runs in front of the rows, workgroup x = 0 publishes it
__global__ __launch_bounds__(256) void mix_up_kernel(const float* logits, const float* correction, int E, int ldl, int groups, int keep, int k,
                                                     const bf16_t* Wg, const bf16_t* Wu, const bf16_t* X, int K, int F, bf16_t* act, float* weights,
                                                     int32_t* idx) {
    ARIA_SMEM_STATIC float lds[4][768];
    const int l = threadIdx.x & 63, w = threadIdx.x >> 6, j = blockIdx.y, tok = blockIdx.z;
    float my_w;
    int my_e;
    const int e = route_group_limited(logits + (long long)tok * ldl, correction, E, groups, keep, k, lds[w], l, j, my_w, my_e);
    if (blockIdx.x == 0 && j == 0 && w == 0 && l < k) {
        weights[tok * k + l] = my_w;
        idx[tok * k + l] = my_e;
    }
    const int n = blockIdx.x * 4 + w;
    if (n >= F) return;
    float acc[2][1] = {{0.f}, {0.f}};
    const long long row = ((long long)e * F + n) * K;
    two_rows<1>(acc, Wg + row, Wu + row, X + (long long)tok * K, K, 1, K, l);
    if (l == 0) act[((long long)tok * k + j) * F + n] = f2bf(silu_fast(acc[0][0]) * acc[1][0]);
}
// down-projections of a token's k experts for two stream columns, their weighted sum, residual and norms
__global__ __launch_bounds__(256) void mix_down_kernel(const bf16_t* Wd, const float* weights, const int32_t* idx, int k, const bf16_t* act, int F, int D,
                                                       RowsOut ro) {
    const int l = threadIdx.x & 63, w = threadIdx.x >> 6, tok = blockIdx.y;
    const int row0 = (blockIdx.x * 4 + w) * 2;
    if (row0 >= D) return;
    float y0 = 0.f, y1 = 0.f;
    for (int j = 0; j < k; ++j) {
        const bf16_t* base = Wd + (long long)idx[tok * k + j] * D * F;
        float acc[2][1] = {{0.f}, {0.f}};
        two_rows<1>(acc, base + (long long)row0 * F, base + (long long)min(row0 + 1, D - 1) * F, act + ((long long)tok * k + j) * F, F, 1, F, l);
        const float wj = weights[tok * k + j];
        y0 += wj * acc[0][0];
        y1 += wj * acc[1][0];
    }
    if (l < 2 && row0 + l < D) stream_step(l ? y1 : y0, ro.post, ro.next, ro.x, ro.h, (long long)tok * D + row0 + l, row0 + l);
}

bool al16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

int shape_ok(const Shape* s) {
    if (!s || s->H <= 0 || s->dn <= 0 || s->dr < 0 || s->dv <= 0 || s->R <= 0 || s->S_cap <= 0) return ARIA_ERR_INVALID;
    if (s->rot < 0 || (s->rot & 1) || s->rot > s->dr || s->dq < s->dn + s->dr || s->dvp < s->dv || s->cw < s->R + s->dr || s->rp < s->R ||
        s->kv_off < s->H * s->dq || s->g_off < s->kv_off + s->R + s->dr || s->ldp < s->g_off + s->H)
        return ARIA_ERR_INVALID;
    if ((s->cw & 63) || (s->rp & 7) || s->rp > s->cw || (s->ldp & 7)) return ARIA_ERR_ALIGN;
    return ARIA_OK;
}

template <class T>
int launch_any(const T* qa, const T* cache, const Shape& s, const int32_t* slot, const int32_t* pos, float* po, float* ml, int64_t n_tok, void* stream) {
    if (s.R > 256 * ANY_COLS) return ARIA_ERR_UNSUPPORTED;
    ARIA_LAUNCH((latent_attn_any_kernel<T>), dim3(unsigned(s.H), unsigned(n_tok)), dim3(256), size_t(s.cw + 264) * 4, stream, qa, cache, s, slot, pos,
                po, ml);
    return aria_check_launch();
}
int mfma_class(const Shape& s) { return tile_attn_class(s.cw, s.R, s.cw); }

}  // namespace

extern "C" {

int aria_latent_rows(void* proj, const AriaLatentShape* s, const int32_t* slot, const int32_t* pos, const float* rope, const float* kv_norm, void* cache,
                     void* packed, int64_t T, int f32, void* stream) {
    if (!proj || !slot || !pos || !rope || !kv_norm || !cache || !packed || T < 0) return ARIA_ERR_INVALID;
    if (const int rc = shape_ok(s)) return rc;
    if (T == 0) return ARIA_OK;
    const dim3 grid(unsigned((T + 3) / 4)), block(256);
    if (f32)
        ARIA_LAUNCH((latent_rows_kernel<float>), grid, block, 0, stream, static_cast<float*>(proj), *s, slot, pos, rope, kv_norm,
                    static_cast<float*>(cache), static_cast<float*>(packed), int(T));
    else
        ARIA_LAUNCH((latent_rows_kernel<bf16_t>), grid, block, 0, stream, static_cast<bf16_t*>(proj), *s, slot, pos, rope, kv_norm,
                    static_cast<bf16_t*>(cache), static_cast<bf16_t*>(packed), int(T));
    return aria_check_launch();
}

int aria_latent_absorb(const void* proj, const AriaLatentShape* s, const int32_t* slot, const int32_t* pos, const float* rope, const float* kv_norm,
                       const void* uk, void* cache, void* qa, int64_t T, int f32, void* stream) {
    if (!proj || !slot || !pos || !rope || !kv_norm || !uk || !cache || !qa || T < 0) return ARIA_ERR_INVALID;
    if (const int rc = shape_ok(s)) return rc;
    if (!al16(uk)) return ARIA_ERR_ALIGN;
    if (T == 0) return ARIA_OK;
    const int NB = T == 1 ? 1 : 4;
    const size_t lds = (size_t(16) * NB * 128 + size_t(NB) * s->dn) * 4;
    if (lds > 160 * 1024) return ARIA_ERR_UNSUPPORTED;
    const dim3 grid(unsigned(s->H * ((s->R + 127) / 128) + 1), unsigned((T + NB - 1) / NB)), block(256);
#define ARIA_ABSORB(T_, B_)                                                                                                                          \
    ARIA_LAUNCH((latent_absorb_kernel<T_, B_>), grid, block, lds, stream, static_cast<const T_*>(proj), *s, slot, pos, rope, kv_norm,                \
                static_cast<const T_*>(uk), static_cast<T_*>(cache), static_cast<T_*>(qa), int(T))
    if (f32) {
        if (NB == 1)
            ARIA_ABSORB(float, 1);
        else
            ARIA_ABSORB(float, 4);
    } else {
        if (NB == 1)
            ARIA_ABSORB(bf16_t, 1);
        else
            ARIA_ABSORB(bf16_t, 4);
    }
#undef ARIA_ABSORB
    return aria_check_launch();
}

int64_t aria_latent_splits(const AriaLatentShape* s, int64_t T, int64_t max_len) {
    if (!s || T <= 0 || !mfma_class(*s)) return 1;
    return tile_attn_splits(s->cw, s->H, s->H, T, max_len);
}

int aria_latent_attn(const void* qa, const void* cache, const AriaLatentShape* s, const int32_t* slot, const int32_t* pos, float* part_o, float* part_ml,
                     int64_t T, int64_t splits, int f32, void* stream) {
    if (!qa || !cache || !slot || !pos || !part_o || !part_ml || T < 0 || splits < 1) return ARIA_ERR_INVALID;
    if (const int rc = shape_ok(s)) return rc;
    if (!al16(qa) || !al16(cache)) return ARIA_ERR_ALIGN;
    if (T == 0) return ARIA_OK;
    if (T > 65535 || splits > MAX_SPLITS) return ARIA_ERR_UNSUPPORTED;
    const int cls = f32 ? 0 : mfma_class(*s);
    if (cls == 0) {
        if (splits != 1) return ARIA_ERR_UNSUPPORTED;
        return f32 ? launch_any(static_cast<const float*>(qa), static_cast<const float*>(cache), *s, slot, pos, part_o, part_ml, T, stream)
                   : launch_any(static_cast<const bf16_t*>(qa), static_cast<const bf16_t*>(cache), *s, slot, pos, part_o, part_ml, T, stream);
    }
    const TileAttn a{static_cast<const bf16_t*>(qa), (long long)(s->H * s->cw), int(s->cw), static_cast<const bf16_t*>(cache), (long long)(s->S_cap * s->cw),
                     0, int(s->cw), int(s->cw), 0, int(s->R), int(s->H), int(s->H), 0, s->scale};
    return launch_tile_attn(a, slot, pos, part_o, part_ml, T, splits, stream);
}

int aria_latent_expand(const float* part_o, const float* part_ml, const AriaLatentShape* s, const void* proj, const void* uv, void* out, int64_t T,
                       int64_t splits, int f32, void* stream) {
    if (!part_o || !part_ml || !proj || !uv || !out || T < 0 || splits < 1) return ARIA_ERR_INVALID;
    if (const int rc = shape_ok(s)) return rc;
    if (!al16(uv)) return ARIA_ERR_ALIGN;
    if (T == 0) return ARIA_OK;
    if (T > 65535 || splits > MAX_SPLITS) return ARIA_ERR_UNSUPPORTED;
    const dim3 grid(unsigned(s->H), unsigned((s->dvp + EXP_ROWS - 1) / EXP_ROWS), unsigned(T)), block(512);
    const size_t lds = size_t(s->rp + MAX_SPLITS) * 4;
    if (f32)
        ARIA_LAUNCH((latent_expand_kernel<float>), grid, block, lds, stream, part_o, part_ml, *s, static_cast<const float*>(proj),
                    static_cast<const float*>(uv), static_cast<float*>(out), int(splits));
    else
        ARIA_LAUNCH((latent_expand_kernel<bf16_t>), grid, block, lds, stream, part_o, part_ml, *s, static_cast<const bf16_t*>(proj),
                    static_cast<const bf16_t*>(uv), static_cast<bf16_t*>(out), int(splits));
    return aria_check_launch();
}

}  // extern "C"

namespace {

struct Scratch {
    float *x, *part_o, *part_ml, *logits, *weights;
    bf16_t *h, *proj, *qa, *ao, *act;
    int32_t* idx;
    int64_t bytes;
};
Scratch layout(const AriaLatentStack& st, const AriaLatentLayer* L, int64_t T, int64_t max_len, char* base) {
    int64_t ldp = 0, qa = 0, ao = 0, act = 0, po = 0, ml = 0, E = 0, k = 0;
    for (int64_t i = 0; i < st.n_layers; ++i) {
        const Shape& s = L[i].mix;
        const int64_t ns = aria_latent_splits(&s, T, max_len);
        ldp = std::max(ldp, s.ldp);
        qa = std::max(qa, s.H * s.cw);
        ao = std::max(ao, s.H * s.dvp);
        po = std::max(po, ns * s.H * s.R);
        ml = std::max(ml, ns * s.H * 2);
        if (L[i].mlp) act = std::max(act, L[i].ff * (L[i].mlp == 2 ? L[i].k : 1));
        if (L[i].mlp == 2) {
            E = std::max(E, (L[i].E + 7) & ~int64_t(7));
            k = std::max(k, L[i].k);
        }
    }
    Scratch z{};
    int64_t at = 0;
    auto take = [&](int64_t bytes) {
        char* p = base + at;
        at += (bytes + 255) & ~int64_t(255);
        return p;
    };
    z.x = reinterpret_cast<float*>(take(4 * T * st.D));
    z.h = reinterpret_cast<bf16_t*>(take(2 * T * st.D));
    z.proj = reinterpret_cast<bf16_t*>(take(2 * T * ldp));
    z.qa = reinterpret_cast<bf16_t*>(take(2 * T * qa));
    z.ao = reinterpret_cast<bf16_t*>(take(2 * T * ao));
    z.act = reinterpret_cast<bf16_t*>(take(2 * T * act));
    z.part_o = reinterpret_cast<float*>(take(4 * T * po));
    z.part_ml = reinterpret_cast<float*>(take(4 * T * ml));
    z.logits = reinterpret_cast<float*>(take(4 * T * E));
    z.weights = reinterpret_cast<float*>(take(4 * T * k));
    z.idx = reinterpret_cast<int32_t*>(take(4 * T * k));
    z.bytes = at;
    return z;
}

template <int MODE>
int rows(const void* W, const bf16_t* X, int64_t ldx, int64_t K, int64_t N, int64_t T, const RowsOut& ro, void* stream) {
    RowsIn in{static_cast<const bf16_t*>(W), nullptr, X, (long long)ldx, int(K), int(N)};
    return launch_rows(RowsPair{{in, in}}, 1, T, LatentRows<MODE>{ro}, stream);
}

}  // namespace

extern "C" {

int64_t aria_latent_decode_scratch(const AriaLatentStack* stack, const AriaLatentLayer* layers, int64_t T, int64_t max_len) {
    if (!stack || !layers || T <= 0 || max_len <= 0) return 0;
    return layout(*stack, layers, T, max_len, nullptr).bytes;
}

int aria_latent_decode(const AriaLatentStack* st, const AriaLatentLayer* L, int64_t T, const int32_t* ids, const int32_t* slot, const int32_t* pos,
                       int64_t max_len, float* logits, void* scratch, int64_t scratch_bytes, void* stream) {
    if (!st || !L || !ids || !slot || !pos || !logits || !scratch || T < 0 || max_len <= 0 || st->n_layers <= 0) return ARIA_ERR_INVALID;
    if (T == 0) return ARIA_OK;
    if ((st->D & 7) || !al16(scratch)) return ARIA_ERR_ALIGN;
    const Scratch z = layout(*st, L, T, max_len, static_cast<char*>(scratch));
    if (scratch_bytes < z.bytes) return ARIA_ERR_INVALID;
    for (int64_t i = 0; i < st->n_layers; ++i) {
        if (const int rc = shape_ok(&L[i].mix)) return rc;
        if (max_len > L[i].mix.S_cap || (L[i].mix.H * L[i].mix.dvp & 7) || (L[i].mlp && (L[i].ff & 7))) return ARIA_ERR_INVALID;
        if (L[i].mlp == 2 && (L[i].E > 256 || L[i].k > 64 || L[i].groups <= 0 || L[i].E % L[i].groups)) return ARIA_ERR_UNSUPPORTED;
    }
    const int64_t D = st->D;
    const AriaDyT none{0.f, nullptr, nullptr};
    int rc = aria_dyt_stream(ids, st->embed, nullptr, nullptr, nullptr, 0, &none, z.x, &st->first, z.h, T, D, 0, 0, stream);
    for (int64_t i = 0; i < st->n_layers && rc == ARIA_OK; ++i) {
        const AriaLatentLayer& y = L[i];
        const Shape& s = y.mix;
        const int64_t ns = aria_latent_splits(&s, T, max_len);
        RowsOut plain{z.proj, (long long)s.ldp, none, none, nullptr, nullptr};
        rc = rows<ROWS_BF16>(y.w_in, z.h, D, D, s.ldp, T, plain, stream);
        if (rc == ARIA_OK) rc = aria_latent_absorb(z.proj, &s, slot, pos, y.rope, y.kv_norm, y.w_uk, y.cache, z.qa, T, 0, stream);
        if (rc == ARIA_OK) rc = aria_latent_attn(z.qa, y.cache, &s, slot, pos, z.part_o, z.part_ml, T, ns, 0, stream);
        if (rc == ARIA_OK) rc = aria_latent_expand(z.part_o, z.part_ml, &s, z.proj, y.w_uv, z.ao, T, ns, 0, stream);
        RowsOut out{nullptr, (long long)D, y.norm1b, y.mlp ? y.norm2 : y.next, z.x, z.h};
        if (rc == ARIA_OK) rc = rows<ROWS_STREAM>(y.w_o, z.ao, s.H * s.dvp, s.H * s.dvp, D, T, out, stream);
        if (rc != ARIA_OK || y.mlp == 0) continue;
        out.post = y.norm2b;
        out.next = y.next;
        if (y.mlp == 1) {
            RowsOut up{z.act, (long long)y.ff, none, none, nullptr, nullptr};
            rc = rows<ROWS_RELU2>(y.w_up, z.h, D, D, y.ff, T, up, stream);
            if (rc == ARIA_OK) rc = rows<ROWS_STREAM>(y.w_down, z.act, y.ff, y.ff, D, T, out, stream);
        } else {
            const int64_t ldl = (y.E + 7) & ~int64_t(7);
            RowsOut lg{z.logits, (long long)ldl, none, none, nullptr, nullptr};
            rc = rows<ROWS_F32>(y.w_router, z.h, D, D, y.E, T, lg, stream);
            if (rc != ARIA_OK) break;
            ARIA_LAUNCH(mix_up_kernel, dim3(unsigned((y.ff + 3) / 4), unsigned(y.k), unsigned(T)), dim3(256), 0, stream, (const float*)z.logits,
                        y.correction, int(y.E), int(ldl), int(y.groups), int(y.keep), int(y.k), static_cast<const bf16_t*>(y.w_gate),
                        static_cast<const bf16_t*>(y.w_up), (const bf16_t*)z.h, int(D), int(y.ff), z.act, z.weights, z.idx);
            ARIA_LAUNCH(mix_down_kernel, dim3(unsigned((D + 7) / 8), unsigned(T)), dim3(256), 0, stream, static_cast<const bf16_t*>(y.w_down),
                        (const float*)z.weights, (const int32_t*)z.idx, int(y.k), (const bf16_t*)z.act, int(y.ff), int(D), out);
            rc = aria_check_launch();
        }
    }
    if (rc != ARIA_OK) return rc;
    RowsOut lo{logits, (long long)st->V, none, none, nullptr, nullptr};
    return rows<ROWS_F32>(st->head, z.h, D, D, st->V, T, lo, stream);
}

}  // extern "C"
