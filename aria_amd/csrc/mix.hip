// The decode step of a stack of linear-attention and chunk-local-attention layers (bf16): one call enqueues every launch of every layer run.
//
// A run whose mixer is linear attention alone takes five launches: input projection, recurrence (with norm weight and output gate), output projection
// with the residual, gate / up with relu, down projection with the residual.  RMS norms without launches of their own: whoever writes the normed quantity
// leaves it without 1 / rms beside partial sums of squares, and the projection that reads it scales its results (rows.h).  The half-sum of two normed
// outputs needs whole rows before it enters the stream: a run with two mixers takes eight launches (input projection with the cache rows, chunk attention,
// recurrence, merge + head norm, both output projections, stream pass, gate / up, down).
#include "linear_step.h"
#include "rows.h"
#include "tile_attn.h"
#include <algorithm>

namespace {
using namespace ad;
typedef AriaChunkShape Chunk;

struct StoreRows {
    static constexpr bool SUMSQ = false;
    bf16_t* out[2];   // per problem
    long long ldo;
    float* sums = nullptr;
    __device__ __forceinline__ float operator()(float v, int tok, int n, int problem) const {
        out[problem][tok * ldo + n] = f2bf(v);
        return 0.f;
    }
};
// input projection of a layer with chunk attention: keys and values also go to the token's cache row
struct StoreRowsAndCache {
    static constexpr bool SUMSQ = false;
    bf16_t *out, *cache;
    Chunk s;
    const int32_t *slot, *pos;
    float* sums = nullptr;
    __device__ __forceinline__ float operator()(float v, int tok, int n, int) const {
        const bf16_t x = f2bf(v);
        out[(long long)tok * s.ldp + n] = x;
        const int kn = n - int(s.k_off), vn = n - int(s.v_off), dq = int(s.dq), dvp = int(s.dvp);
        const bool key = kn >= 0 && kn < s.G * dq;
        if (key || (vn >= 0 && vn < s.G * dvp)) {
            const int g = key ? kn / dq : vn / dvp, c = key ? kn % dq : dq + vn % dvp;
            cache[((slot[tok] * s.G + g) * s.cap + pos[tok] % int(s.size)) * (dq + dvp) + c] = x;
        }
        return 0.f;
    }
};
// x += mult v (+ embedding rows); h = x times the next norm's weight, 1 / rms left to the reader
struct ResidualRows {
    static constexpr bool SUMSQ = true;
    float *x, *sums;
    bf16_t* h;
    const float* w;
    long long D;
    float mult, scale;
    const int32_t* ids;   // NULL: no embedding
    const bf16_t* table;
    __device__ __forceinline__ float operator()(float v, int tok, int n, int) const {
        const long long at = tok * D + n;
        float xn = x[at] + mult * v;
        if (ids) xn += scale * bf2f(table[ids[tok] * D + n]);
        x[at] = xn;
        h[at] = f2bf(xn * w[n]);
        return xn * xn;
    }
};
struct ReluGate {
    static constexpr bool SUMSQ = false;
    bf16_t* act;
    long long ff;
    float* sums = nullptr;
    __device__ __forceinline__ float operator()(float g, float u, int tok, int n) const {
        act[tok * ff + n] = f2bf(fmaxf(g, 0.f) * u);
        return 0.f;
    }
    __device__ __forceinline__ float operator()(float, int, int, int) const { return 0.f; }
};
struct CappedLogits {
    static constexpr bool SUMSQ = false;
    float* out;
    long long V;
    float cap;
    float* sums = nullptr;
    __device__ __forceinline__ float operator()(float v, int tok, int n, int) const {
        out[tok * V + n] = softcap(v, cap);
        return 0.f;
    }
};

// a wave per (token, query head): merge of the attention's splits; then a wave per (token, linear head): RMS norm and gate in place
__global__ __launch_bounds__(256) void mix_finish_kernel(const float* part_o, const float* part_ml, int splits, int H, int dvp, bf16_t* ao, bf16_t* lo, const bf16_t* proj,
                                                         AriaLinearShape r, long long g_off, const float* norm, float eps, int n_tok) {
    const int l = threadIdx.x & 63, item = blockIdx.x * 4 + (threadIdx.x >> 6), n_attn = n_tok * H;
    if (item < n_attn) {
        const int tok = item / H, h = item % H;
        float m = -INFINITY, sum = 0.f;
        if (l < splits) {
            const float* ml = part_ml + (((long long)tok * splits + l) * H + h) * 2;
            m = ml[0];
            sum = ml[1];
        }
        const float mx = wave_max_bcast(m);
        const float f = sum > 0.f ? exp2f(m - mx) : 0.f;
        const float wt = f / wave_sum_bcast(sum * f);   // lane = split
        const float* po = part_o + ((long long)tok * splits * H + h) * dvp;
        float acc[4] = {0.f, 0.f, 0.f, 0.f};
        for (int j = 0; j < splits; j += 8) {           // (a split without rows left its slab unwritten: selected away, not multiplied)
            float x[8][4];
#pragma unroll
            for (int u = 0; u < 8; ++u)
#pragma unroll
                for (int i = 0; i < 4; ++i) x[u][i] = po[(long long)min(j + u, splits - 1) * H * dvp + min(l + 64 * i, dvp - 1)];
#pragma unroll
            for (int u = 0; u < 8; ++u) {
                const float wj = j + u < splits ? shfl(wt, j + u) : 0.f;
#pragma unroll
                for (int i = 0; i < 4; ++i) acc[i] += wj != 0.f ? wj * x[u][i] : 0.f;
            }
        }
#pragma unroll
        for (int i = 0; i < 4; ++i)
            if (l + 64 * i < dvp) ao[(long long)item * dvp + l + 64 * i] = f2bf(acc[i]);
        return;
    }
    const int it2 = item - n_attn, rh = int(r.H), cols = int(r.dvp);
    if (it2 >= n_tok * rh) return;
    const int tok = it2 / rh, h = it2 % rh;
    bf16_t* o = lo + (long long)it2 * cols;
    const bf16_t* gate = proj + tok * r.ldp + g_off + (long long)h * cols;
    float ss = 0.f;
    for (int c = l * 8; c < cols; c += 512) {
        float v[8];
        ld8(o + c, v);
#pragma unroll
        for (int e = 0; e < 8; ++e) ss += v[e] * v[e];
    }
    const float rs = 1.f / sqrtf(wave_sum_bcast(ss) / float(r.dv) + eps);
    for (int c = l * 8; c < cols; c += 512) {
        float v[8], g[8], w[8];
        ld8(o + c, v);
        ld8(gate + c, g);
        ld8(norm + c, w);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = v[e] * rs * w[e] * silu_exact(g[e]);
        st8(o + c, v);
    }
}

struct Scratch {
    float *x, *sums, *lsums, *part_o, *part_ml;
    bf16_t *h, *proj, *ao, *lo, *y, *act;
    int64_t bytes;
};
int64_t keys_of(const Chunk& s, int64_t max_len) { return std::min(s.size, max_len); }
int64_t splits_of(const Chunk& s, int64_t T, int64_t max_len) { return tile_attn_splits(s.dq + s.dvp, s.H, s.H / s.G, T, keys_of(s, max_len)); }
bool tile_shape_ok(const Chunk& s) { return tile_attn_class(s.dq, s.dvp, s.dq + s.dvp) && s.dvp <= 256; }
TileAttn tile_args(const Chunk& s, const bf16_t* proj, const void* ring) {
    const int cw = int(s.dq + s.dvp);
    return TileAttn{proj + s.q_off, (long long)s.ldp, int(s.dq), static_cast<const bf16_t*>(ring), (long long)(s.G * s.cap * cw), (long long)(s.cap * cw), cw, int(s.dq),
                    int(s.dq), int(s.dvp), int(s.H), int(s.H / s.G), int(std::min<int64_t>(s.size, INT32_MAX)), s.scale};
}
Scratch layout(const AriaMixStack& st, const AriaMixLayer* L, int64_t T, int64_t max_len, char* base) {
    int64_t ldp = 0, ao = 0, lo = 0, ls = 0, act = 0, po = 0, ml = 0;
    for (int64_t i = 0; i < st.n_runs; ++i) {
        const AriaLinearShape& r = L[i].right;
        ldp = std::max(ldp, r.ldp);
        lo = std::max(lo, r.H * r.dvp);
        ls = std::max(ls, r.H * step_blocks(r, T));
        if (L[i].norm2) act = std::max(act, L[i].ff);
        if (L[i].kind) {
            const Chunk& s = L[i].left;
            const int64_t ns = splits_of(s, T, max_len);
            ao = std::max(ao, s.H * s.dvp);
            po = std::max(po, ns * s.H * s.dvp);
            ml = std::max(ml, ns * s.H * 2);
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
    z.sums = reinterpret_cast<float*>(take(4 * T * rows_parts(T, st.D)));
    z.lsums = reinterpret_cast<float*>(take(4 * T * ls));
    z.part_o = reinterpret_cast<float*>(take(4 * T * po));
    z.part_ml = reinterpret_cast<float*>(take(4 * T * ml));
    z.h = reinterpret_cast<bf16_t*>(take(2 * T * st.D));
    z.proj = reinterpret_cast<bf16_t*>(take(2 * T * ldp));
    z.ao = reinterpret_cast<bf16_t*>(take(2 * T * ao));
    z.lo = reinterpret_cast<bf16_t*>(take(2 * T * lo));
    z.y = reinterpret_cast<bf16_t*>(take(2 * 2 * T * st.D));
    z.act = reinterpret_cast<bf16_t*>(take(2 * T * act));
    z.bytes = at;
    return z;
}
int layer_ok(const AriaMixLayer& y, int64_t max_len) {
    const AriaLinearShape& r = y.right;
    if (!y.w_in || !y.w_o || !y.norm || !y.state || !y.next || (y.norm2 && (!y.w_gate || !y.w_up || !y.w_down || y.ff <= 0 || (y.ff & 7)))) return ARIA_ERR_INVALID;
    if (r.H <= 0 || r.dp <= 0 || r.dvp <= 0 || r.dv <= 0 || (r.dp & 7) || (r.dvp & 7) || (r.ldp & 7) || (!r.decay && (!r.a2 || !r.a_bias || r.rank <= 0 || (r.rank & 7))))
        return ARIA_ERR_INVALID;
    if (r.q_off + r.H * r.dp > r.ldp || r.k_off + r.H * r.dp > r.ldp || r.v_off + r.H * r.dvp > r.ldp || y.g_off + r.H * r.dvp > r.ldp || r.a_off + r.rank > r.ldp)
        return ARIA_ERR_INVALID;
    if (r.dp > 1024) return ARIA_ERR_UNSUPPORTED;
    if (y.kind == 0) return ARIA_OK;
    const Chunk& s = y.left;
    if (!y.w_o_left || !y.out_left || !y.out_right || !y.ring || s.H <= 0 || s.G <= 0 || s.H % s.G || s.size <= 0 || keys_of(s, max_len) > s.cap || s.ldp != r.ldp ||
        s.q_off + s.H * s.dq > s.ldp || s.k_off + s.G * s.dq > s.ldp || s.v_off + s.G * s.dvp > s.ldp || (s.q_off & 7) || (s.dq & 7) || (s.dvp & 7))
        return ARIA_ERR_INVALID;
    return tile_shape_ok(s) ? ARIA_OK : ARIA_ERR_UNSUPPORTED;
}

}  // namespace

extern "C" {

int64_t aria_chunk_decode_scratch(const AriaChunkShape* s, int64_t T, int64_t max_len) {
    if (!s || T <= 0 || max_len <= 0 || s->H <= 0 || s->G <= 0 || !tile_shape_ok(*s)) return 0;
    return 4 * T * splits_of(*s, T, max_len) * s->H * (s->dvp + 2);
}

int aria_chunk_decode(const void* proj, const void* cache, const AriaChunkShape* s, const int32_t* slot, const int32_t* pos, int64_t max_len, void* out, int64_t T,
                      void* scratch, int64_t scratch_bytes, void* stream) {
    if (!proj || !cache || !s || !slot || !pos || !out || !scratch || T < 0 || max_len <= 0 || s->H <= 0 || s->G <= 0 || s->H % s->G || s->size <= 0 ||
        keys_of(*s, max_len) > s->cap || s->q_off + s->H * s->dq > s->ldp)
        return ARIA_ERR_INVALID;
    if ((s->ldp & 7) || (s->q_off & 7) || (reinterpret_cast<uintptr_t>(proj) & 15) || (reinterpret_cast<uintptr_t>(cache) & 15)) return ARIA_ERR_ALIGN;
    if (!tile_shape_ok(*s) || T > 65535) return ARIA_ERR_UNSUPPORTED;
    if (T == 0) return ARIA_OK;
    if (scratch_bytes < aria_chunk_decode_scratch(s, T, max_len)) return ARIA_ERR_INVALID;
    const int64_t ns = splits_of(*s, T, max_len);
    float *po = static_cast<float*>(scratch), *ml = po + T * ns * s->H * s->dvp;
    if (const int rc = launch_tile_attn(tile_args(*s, static_cast<const bf16_t*>(proj), cache), slot, pos, po, ml, T, ns, stream)) return rc;
    ARIA_LAUNCH(mix_finish_kernel, dim3(unsigned((T * s->H + 3) / 4)), dim3(256), 0, stream, (const float*)po, (const float*)ml, int(ns), int(s->H), int(s->dvp),
                static_cast<bf16_t*>(out), static_cast<bf16_t*>(nullptr), static_cast<const bf16_t*>(nullptr), AriaLinearShape{}, 0ll,
                static_cast<const float*>(nullptr), 0.f, int(T));
    return aria_check_launch();
}

int64_t aria_mix_decode_scratch(const AriaMixStack* st, const AriaMixLayer* runs, int64_t T, int64_t max_len) {
    if (!st || !runs || T <= 0 || max_len <= 0) return 0;
    return layout(*st, runs, T, max_len, nullptr).bytes;
}

int aria_mix_decode(const AriaMixStack* st, const AriaMixLayer* L, int64_t T, const int32_t* ids, const int32_t* slot, const int32_t* pos, int64_t max_len,
                    float* logits, void* scratch, int64_t scratch_bytes, void* stream) {
    if (!st || !L || !ids || !slot || !pos || !logits || !scratch || T < 0 || max_len <= 0 || st->n_runs <= 0) return ARIA_ERR_INVALID;
    if (T == 0) return ARIA_OK;
    if ((st->D & 7) || (reinterpret_cast<uintptr_t>(scratch) & 15)) return ARIA_ERR_ALIGN;
    const Scratch z = layout(*st, L, T, max_len, static_cast<char*>(scratch));
    if (scratch_bytes < z.bytes || T > 65535) return ARIA_ERR_INVALID;
    for (int64_t i = 0; i < st->n_runs; ++i)
        if (const int rc = layer_ok(L[i], max_len)) return rc;
    const int64_t D = st->D;
    auto bf = [](const void* p) { return static_cast<const bf16_t*>(p); };
    AriaRmsStream rs{ids, st->embed, st->embedding_scale, st->mult, st->eps, st->n, D, nullptr, nullptr, nullptr, nullptr, z.x, st->first, z.h};
    int rc = aria_rms_stream(&rs, T, D, 0, stream);
    const int parts = rows_parts(T, D);
    bool scaled = true;   // h carries its 1 / rms
    auto input = [&](const void* W, const void* W2, int64_t N) {
        RowsIn in{bf(W), bf(W2), z.h, (long long)D, int(D), int(N)};
        if (!scaled) {
            in.sq = z.sums;
            in.sq_n = parts;
            in.inv_n = 1.f / float(st->n);
            in.eps = st->eps;
        }
        return in;
    };
    for (int64_t i = 0; i < st->n_runs && rc == ARIA_OK; ++i) {
        const AriaMixLayer& y = L[i];
        const AriaLinearShape& r = y.right;
        // the stream behind a sublayer: `last` of the run?
        auto residual = [&](bool last) {
            const bool emb = last && y.next_embedding;
            return ResidualRows{z.x, z.sums, z.h, last ? y.next : y.norm2, (long long)D, st->mult, st->embedding_scale, emb ? ids : nullptr, bf(st->embed)};
        };
        const RowsIn in = input(y.w_in, nullptr, r.ldp);
        if (y.kind == 0) {
            rc = launch_rows(RowsPair{{in, in}}, 1, T, StoreRows{{z.proj, z.proj}, (long long)r.ldp}, stream);
            if (rc == ARIA_OK) rc = launch_step<bf16_t>(z.proj, r, y.state, slot, pos, nullptr, T, z.lo, StepOut{z.lsums, y.norm, (long long)y.g_off}, stream);
            RowsIn o{bf(y.w_o), nullptr, z.lo, (long long)(r.H * r.dvp), int(r.H * r.dvp), int(D)};
            o.sq = z.lsums;
            o.sq_n = int(r.H * step_blocks(r, T));
            o.inv_n = 1.f / float(r.H * r.dv);
            o.eps = st->eps;
            if (rc == ARIA_OK) rc = launch_rows(RowsPair{{o, o}}, 1, T, residual(!y.norm2), stream);
            scaled = false;
        } else {
            const Chunk& s = y.left;
            const int64_t ns = splits_of(s, T, max_len);
            rc = launch_rows(RowsPair{{in, in}}, 1, T, StoreRowsAndCache{z.proj, static_cast<bf16_t*>(y.ring), s, slot, pos}, stream);
            if (rc == ARIA_OK) rc = launch_tile_attn(tile_args(s, z.proj, y.ring), slot, pos, z.part_o, z.part_ml, T, ns, stream);
            if (rc == ARIA_OK) rc = launch_step<bf16_t>(z.proj, r, y.state, slot, pos, nullptr, T, z.lo, StepOut{}, stream);
            if (rc != ARIA_OK) break;
            ARIA_LAUNCH(mix_finish_kernel, dim3(unsigned((T * (s.H + r.H) + 3) / 4)), dim3(256), 0, stream, (const float*)z.part_o, (const float*)z.part_ml, int(ns),
                        int(s.H), int(s.dvp), z.ao, z.lo, (const bf16_t*)z.proj, r, (long long)y.g_off, y.norm, st->eps, int(T));
            rc = aria_check_launch();
            const RowsIn left{bf(y.w_o_left), nullptr, z.ao, (long long)(s.H * s.dvp), int(s.H * s.dvp), int(D)};
            const RowsIn right{bf(y.w_o), nullptr, z.lo, (long long)(r.H * r.dvp), int(r.H * r.dvp), int(D)};
            bf16_t* y2 = z.y + T * D;
            if (rc == ARIA_OK) rc = launch_rows(RowsPair{{left, right}}, 2, T, StoreRows{{z.y, y2}, (long long)D}, stream);
            const bool last = !y.norm2, emb = last && y.next_embedding;
            AriaRmsStream a{emb ? ids : nullptr, st->embed, st->embedding_scale, st->mult, st->eps, st->n, D, z.y, y2, y.out_left, y.out_right, z.x,
                            last ? y.next : y.norm2, z.h};
            if (rc == ARIA_OK) rc = aria_rms_stream(&a, T, D, 0, stream);
            scaled = true;
        }
        if (rc != ARIA_OK || !y.norm2) continue;
        rc = launch_row_pairs(input(y.w_gate, y.w_up, y.ff), T, ReluGate{z.act, (long long)y.ff}, stream);
        const RowsIn down{bf(y.w_down), nullptr, z.act, (long long)y.ff, int(y.ff), int(D)};
        if (rc == ARIA_OK) rc = launch_rows(RowsPair{{down, down}}, 1, T, residual(true), stream);
        scaled = false;
    }
    if (rc != ARIA_OK) return rc;
    const RowsIn head = input(st->head, nullptr, st->V);
    return launch_rows(RowsPair{{head, head}}, 1, T, CappedLogits{logits, (long long)st->V, st->cap}, stream);
}

}  // extern "C"
