// Chunk-local grouped-query attention: positions form chunks of `size`, a query sees its own chunk up to itself.  The cache of a sequence is therefore
// ONE chunk, position p in row p % size, and the keys a decode step sees are the rows 0 .. p % size.  Whole prompts run the flash kernel of attn.hip
// with every chunk as a sequence of its own; the kernel here takes any widths and any cut of the sequences.
#include "elem.h"

namespace {
using namespace ad;
typedef AriaChunkShape Shape;

// One workgroup per (head, token): a thread per key of a 256-key tile, then a thread per value column.  Key j of the token's chunk is a row of this
// call when the sequence's rows here reach back to it, else a cache row.
constexpr int ANY_COLS = 8;   // value columns per thread: dvp <= 2048
template <class T>
__global__ __launch_bounds__(256) void chunk_attn_any_kernel(const T* proj, const T* cache, Shape s, const int32_t* slot, const int32_t* pos, const int32_t* seq,
                                                             const int32_t* cu, T* out) {
    ARIA_DYN_SMEM(smem);
    float* sq = reinterpret_cast<float*>(smem);   // [dq]
    float* sp = sq + s.dq;                        // [256]
    float* sr = sp + 256;                         // [8]
    const int t = threadIdx.x, l = t & 63, w = t >> 6, h = blockIdx.y, tok = blockIdx.x;
    const int g = h / int(s.H / s.G), p0 = pos[tok], size = int(s.size), first = p0 / size * size;   // keys: positions first .. p0
    const int start = p0 - (tok - cu[seq[tok]]);                                                     // the sequence's first position of this call
    const long long cw = s.dq + s.dvp;
    const T* ring = cache + ((long long)slot[tok] * s.G + g) * s.cap * cw;
    auto key = [&](int j) __attribute__((always_inline)) -> const T* {
        return j >= start ? proj + (long long)(tok - (p0 - j)) * s.ldp + s.k_off + g * s.dq : ring + (long long)(j - first) * cw;
    };
    auto value = [&](int j) __attribute__((always_inline)) -> const T* {
        return j >= start ? proj + (long long)(tok - (p0 - j)) * s.ldp + s.v_off + g * s.dvp : ring + (long long)(j - first) * cw + s.dq;
    };
    const T* q = proj + (long long)tok * s.ldp + s.q_off + h * s.dq;
    for (int i = t; i < s.dq; i += 256) sq[i] = ldf(q + i);
    float acc[ANY_COLS], m = -INFINITY, lsum = 0.f;
#pragma unroll
    for (int j = 0; j < ANY_COLS; ++j) acc[j] = 0.f;
    const float scale2 = s.scale * 1.4426950408889634f;
    sync();
    for (int k0 = first; k0 <= p0; k0 += 256) {
        float x = -INFINITY;
        if (k0 + t <= p0) {
            const T* row = key(k0 + t);
            float d = 0.f;
            for (int c = 0; c < s.dq; c += 8) {
                float v[8];
                ld8(row + c, v);
#pragma unroll
                for (int e = 0; e < 8; ++e) d += v[e] * sq[c + e];
            }
            x = d * scale2;
        }
        const float mx = wave_max(x);
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
        const int n = min(256, p0 + 1 - k0);
#pragma unroll
        for (int j = 0; j < ANY_COLS; ++j) {
            const int c = t + 256 * j;
            if (c < s.dvp) {
                float a = acc[j] * alpha;
                for (int i = 0; i < n; ++i) a += sp[i] * ldf(value(k0 + i) + c);
                acc[j] = a;
            }
        }
        sync();
    }
    T* o = out + ((long long)tok * s.H + h) * s.dvp;
#pragma unroll
    for (int j = 0; j < ANY_COLS; ++j)
        if (t + 256 * j < s.dvp) stf(o + t + 256 * j, acc[j] / lsum);
}

// keys and values of a call's tokens into the cache: a wave per token, 8 columns a lane
template <class T>
__global__ __launch_bounds__(256) void chunk_rows_kernel(const T* proj, T* cache, Shape s, const int32_t* slot, const int32_t* pos, const int32_t* seq,
                                                         const int32_t* cu, int n_tok) {
    const int l = threadIdx.x & 63, t = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (t >= n_tok) return;
    const int last = cu[seq[t] + 1] - 1, size = int(s.size);
    if (last - t >= size) return;   // a later token of this call takes the row
    const int kc = int(s.dq) >> 3, vc = int(s.dvp) >> 3;
    const long long cw = s.dq + s.dvp, row = pos[t] % size;
    const T* p = proj + (long long)t * s.ldp;
    for (int i = l; i < s.G * (kc + vc); i += 64) {
        const int g = i / (kc + vc), c = i % (kc + vc);
        const T* src = c < kc ? p + s.k_off + g * s.dq + c * 8 : p + s.v_off + g * s.dvp + (c - kc) * 8;
        float v[8];
        ld8(src, v);
        st8(cache + (((long long)slot[t] * s.G + g) * s.cap + row) * cw + c * 8, v);
    }
}

bool al16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }
int shape_ok(const Shape* s) {
    if (!s || s->H <= 0 || s->G <= 0 || s->H % s->G || s->dq <= 0 || s->dvp <= 0 || s->size <= 0 || s->cap <= 0) return ARIA_ERR_INVALID;
    if (s->q_off + s->H * s->dq > s->ldp || s->k_off + s->G * s->dq > s->ldp || s->v_off + s->G * s->dvp > s->ldp) return ARIA_ERR_INVALID;
    if ((s->dq & 7) || (s->dvp & 7) || (s->ldp & 7) || (s->q_off & 7) || (s->k_off & 7) || (s->v_off & 7)) return ARIA_ERR_ALIGN;
    return ARIA_OK;
}

}  // namespace

extern "C" {

int aria_chunk_attn_any(const void* proj, const void* cache, const AriaChunkShape* s, const int32_t* slot, const int32_t* pos, const int32_t* seq,
                        const int32_t* cu, void* out, int64_t T, int f32, void* stream) {
    if (!proj || !cache || !slot || !pos || !seq || !cu || !out || T < 0) return ARIA_ERR_INVALID;
    if (const int rc = shape_ok(s)) return rc;
    if (!al16(proj) || !al16(cache)) return ARIA_ERR_ALIGN;
    if (s->dvp > 256 * ANY_COLS || s->H > 65535 || s->dq > 32768) return ARIA_ERR_UNSUPPORTED;
    if (T == 0) return ARIA_OK;
    const dim3 grid(unsigned(T), unsigned(s->H)), block(256);
    const size_t lds = size_t(s->dq + 264) * 4;
    if (f32)
        ARIA_LAUNCH((chunk_attn_any_kernel<float>), grid, block, lds, stream, static_cast<const float*>(proj), static_cast<const float*>(cache), *s, slot,
                    pos, seq, cu, static_cast<float*>(out));
    else
        ARIA_LAUNCH((chunk_attn_any_kernel<bf16_t>), grid, block, lds, stream, static_cast<const bf16_t*>(proj), static_cast<const bf16_t*>(cache), *s, slot,
                    pos, seq, cu, static_cast<bf16_t*>(out));
    return aria_check_launch();
}

int aria_chunk_rows(const void* proj, void* cache, const AriaChunkShape* s, const int32_t* slot, const int32_t* pos, const int32_t* seq, const int32_t* cu,
                    int64_t T, int f32, void* stream) {
    if (!proj || !cache || !slot || !pos || !seq || !cu || T < 0) return ARIA_ERR_INVALID;
    if (const int rc = shape_ok(s)) return rc;
    if (!al16(proj) || !al16(cache)) return ARIA_ERR_ALIGN;
    if (T == 0) return ARIA_OK;
    const dim3 grid(unsigned((T + 3) / 4)), block(256);
    if (f32)
        ARIA_LAUNCH((chunk_rows_kernel<float>), grid, block, 0, stream, static_cast<const float*>(proj), static_cast<float*>(cache), *s, slot, pos, seq, cu,
                    int(T));
    else
        ARIA_LAUNCH((chunk_rows_kernel<bf16_t>), grid, block, 0, stream, static_cast<const bf16_t*>(proj), static_cast<bf16_t*>(cache), *s, slot, pos, seq,
                    cu, int(T));
    return aria_check_launch();
}

}  // extern "C"
