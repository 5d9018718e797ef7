// Grouped-query attention on a window with kept first tokens: query head h reads key / value head h / (heads / kv_heads).
// Queries and keys may be RMS-normed per head (shared weights) and are rotated; keys are cached after both, in one row per
// position: [kv_heads][dnp] keys | [kv_heads][dvp] values, lengths rounded up to 8 with zeros.
//   position i sees j <= i when i - j < window or j < keep; a sink adds exp(sink_h) to a head's denominator
// The cache of a layer is a ring of keep + window rows whose first `keep` stay (fh_ring_row), so its live rows are exactly
// the positions the next token sees.
#pragma once
#include "fh_window_attn.h"

struct FhGqa {
    int heads = 0, kv_heads = 1, dim = 0, vdim = 0;
    int dnp = 0, dvp = 0;                    // dim, vdim rounded up to 8
    int col_q = 0, col_k = 0, col_v = 0;     // columns of a projection row
    int window = 0, keep = 0;                // window 0: all earlier positions
    float scale = 1.f, eps = 0.f, out_scale = 1.f;
    const float *q_norm = nullptr, *k_norm = nullptr; // [dim] or NULL
    const float *sink = nullptr;             // [heads] or NULL
    const float *cos_t = nullptr, *sin_t = nullptr; // [positions, pairs]
    int pairs = 0, halves = 0;               // fh_rotated
};
static inline int fh_gqa_row(const FhGqa &a) { return a.kv_heads * (a.dnp + a.dvp); }
// rows of a portion's work arrays: the kept positions ahead of the window of its first token, that window, the portion
static inline int fh_gqa_lo(const FhGqa &a, int pos) { return a.window && pos > a.window - 1 ? pos - (a.window - 1) : 0; }
static inline int fh_gqa_kept(const FhGqa &a, int pos) { return a.keep < fh_gqa_lo(a, pos) ? a.keep : fh_gqa_lo(a, pos); }
static inline int fh_gqa_keys(const FhGqa &a, int s, int pos) { return fh_gqa_kept(a, pos) + pos + s - fh_gqa_lo(a, pos); }

struct FhGqaWork {
    void *kn, *vr;   // [keys, kv_heads * dnp], [keys, kv_heads * dvp]
    void *vt;        // [kv_heads * vdim, ldt]
    void *q;         // [s, heads, fh_window_dq]
    int64_t ldt;
};
// One portion of s tokens at position pos: o rows of stride ldo, heads * vdim values times out_scale, zeros up to kp.
fh_status fh_gqa_prefill(fh_device *dev, int dtype, const FhGqa &a, fh_kvcache *cache, const float *proj, int64_t ldp, int s, int pos,
                         const FhGqaWork &w, void *o, int ldo, int kp);

// ---------------------------------------------------------------- decode step
enum { FH_GQA_HEADS = 4, FH_GQA_MAX_SPLITS = 32 }; // query heads of a workgroup, parts of the cache
static inline int fh_gqa_splits(const fh_kvcache *c) {
    const int n = c->capacity / 32;
    return n < 1 ? 1 : n > FH_GQA_MAX_SPLITS ? FH_GQA_MAX_SPLITS : n;
}
static inline int fh_gqa_groups(const FhGqa &a) { return (a.heads / a.kv_heads + FH_GQA_HEADS - 1) / FH_GQA_HEADS; }
static inline int fh_gqa_blocks(const FhGqa &a, int splits) { return splits * a.kv_heads * fh_gqa_groups(a); }
static inline size_t fh_gqa_part_floats(const FhGqa &a) { return (size_t)a.heads * FH_GQA_MAX_SPLITS * (a.dvp + 2); }
// LDS of a workgroup of fh_gqa_step, bytes
static inline size_t fh_gqa_lds(const FhGqa &a) {
    const int work = a.dnp > 4 * (a.dvp + 2) ? a.dnp : 4 * (a.dvp + 2);
    return (size_t)(FH_GQA_HEADS * a.dnp + a.dnp + a.dvp + FH_GQA_HEADS * work) * 4;
}

#ifdef __HIPCC__
#include "fh_recurrent.h"
// One head of at most 256 values in a wavefront's registers: value, norm weight, and the cosine and sine of its pair.  The
// request and the work are apart, so that several heads' requests can be on their way at once.
struct FhHead { float x[4], w[4], c[4], s[4]; };
__device__ __forceinline__ void fh_head_load(const FhGqa &a, const float *raw, const float *w, const float *ct, const float *st, FhHead &h) {
    const int lane = threadIdx.x & 63;
#pragma unroll
    for (int j = 0; j < 4; j++) {
        const int i = lane + 64 * j, p = a.halves ? i < a.pairs ? i : i - a.pairs : i >> 1;
        const bool ok = i < a.dim, turn = ok && i < 2 * a.pairs;
        h.x[j] = ok ? raw[i] : 0.f;
        h.w[j] = ok && w ? w[i] : 1.f;
        h.c[j] = turn ? ct[p] : 1.f;
        h.s[j] = turn ? st[p] : 0.f;
    }
}
// RMS norm (norm 0: none) and rotation: dst [pad] times mul, through `tmp` [dim] (LDS).
__device__ __forceinline__ void fh_head_rotate(const FhGqa &a, FhHead &h, int norm, float mul, float *tmp, float *dst, int pad) {
    const int lane = threadIdx.x & 63;
    if (norm) {
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < 4; j++) ss = fmaf(h.x[j], h.x[j], ss);
        const float inv = 1.0f / sqrtf(fh_wave_sum(ss) / (float)a.dim + a.eps);
#pragma unroll
        for (int j = 0; j < 4; j++) h.x[j] *= inv * h.w[j];
    }
#pragma unroll
    for (int j = 0; j < 4; j++)
        if (lane + 64 * j < a.dim) tmp[lane + 64 * j] = h.x[j];
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
#pragma unroll
    for (int j = 0; j < 4; j++) {
        const int i = lane + 64 * j;
        if (i >= pad) break;
        float v = 0.f;
        if (i < a.dim) {
            v = h.x[j];
            if (i < 2 * a.pairs) {
                const bool second = a.halves ? i >= a.pairs : i & 1;
                const float o = tmp[a.halves ? second ? i - a.pairs : i + a.pairs : i ^ 1];
                v = v * h.c[j] + (second ? o : -o) * h.s[j];
            }
        }
        dst[i] = v * mul;
    }
}

// Workgroup b of fh_gqa_blocks: up to FH_GQA_HEADS query heads of one key head against one part of the cache.  The 16 lanes
// of a DPP row take one cached row, pieces of 8 elements; NP pieces per lane (dim and vdim at most 128 NP).  The row of this
// position is computed here, used from the LDS and stored by one of the workgroups that need it.
template <typename T, int NP>
__device__ __forceinline__ void fh_gqa_step(const FhGqa &a, const float *proj, T *ring, int cap, int pos, int splits, int b,
                                            float *__restrict__ part, float *lds) {
    constexpr int HB = FH_GQA_HEADS;
    const float LOG2E = 1.4426950408889634f;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, l16 = lane & 15, rg = tid >> 4;
    const int rep = a.heads / a.kv_heads, hg = b % ((rep + HB - 1) / HB), bb = b / ((rep + HB - 1) / HB);
    const int split = bb % splits, kh = bb / splits, h0 = kh * rep + hg * HB, nh = rep - hg * HB < HB ? rep - hg * HB : HB;
    const int n = pos + 1 < cap ? pos + 1 : cap, mine = fh_ring_row(pos, cap, a.keep);
    const int per = ((n + splits - 1) / splits + 15) / 16 * 16;
    const int k0 = split * per, k1 = k0 + per < n ? k0 + per : n;
    const int row = a.kv_heads * (a.dnp + a.dvp), nk = a.dnp / 8, nv = a.dvp / 8;
    const bool own = mine >= k0 && mine < k1;
    float *sq = lds, *sk = sq + HB * a.dnp, *sv = sk + a.dnp, *od = sv + a.dvp;
    const T *kp_ = ring + kh * a.dnp, *vp_ = ring + a.kv_heads * a.dnp + kh * a.dvp;
    constexpr int U = NP == 1 ? 4 : 2; // rows of a lane group on their way
    FhPiece<T> nx[U][NP], ny[U][NP];
    auto fetch = [&](int k, FhPiece<T> *x, FhPiece<T> *y) {
        const bool in = k < k1;
#pragma unroll
        for (int i = 0; i < NP; i++) {
            x[i] = in && l16 + 16 * i < nk ? fh_ld_piece(kp_ + (int64_t)k * row + (l16 + 16 * i) * 8) : fh_zero_piece<T>();
            y[i] = in && l16 + 16 * i < nv ? fh_ld_piece(vp_ + (int64_t)k * row + (l16 + 16 * i) * 8) : fh_zero_piece<T>();
        }
    };
#pragma unroll
    for (int u = 0; u < U; u++) fetch(k0 + rg + 16 * u, nx[u], ny[u]); // before the query is worked on; this position's row is replaced below
    const float *ct = a.cos_t + (int64_t)pos * a.pairs, *st = a.sin_t + (int64_t)pos * a.pairs;
    FhHead hq, hk;
    float hv = 0.f;
    if (wave < nh) fh_head_load(a, proj + a.col_q + (h0 + wave) * a.dim, a.q_norm, ct, st, hq);
    if (own) {
        if (wave == 0) fh_head_load(a, proj + a.col_k + kh * a.dim, a.k_norm, ct, st, hk);
        if (tid < a.vdim) hv = proj[a.col_v + kh * a.vdim + tid];
    }
    if (wave < nh) fh_head_rotate(a, hq, a.q_norm != nullptr, a.scale * LOG2E, od + wave * a.dnp, sq + wave * a.dnp, a.dnp);
    if (own && wave == 0) fh_head_rotate(a, hk, a.k_norm != nullptr, 1.f, od, sk, a.dnp);
    __syncthreads();
    if (own) {
        for (int i = tid; i < a.dnp; i += 256) sk[i] = fh_up(fh_to<T>(sk[i])); // as the cache holds it
        for (int i = tid; i < a.dvp; i += 256) sv[i] = fh_up(fh_to<T>(hv)); // dvp is at most 256
        if (hg == 0) {
            T *dst = ring + (int64_t)mine * row;
            for (int i = tid; i < a.dnp; i += 256) dst[kh * a.dnp + i] = fh_to<T>(sk[i]);
            for (int i = tid; i < a.dvp; i += 256) dst[a.kv_heads * a.dnp + kh * a.dvp + i] = fh_to<T>(sv[i]);
        }
    }
    __syncthreads();
    float q[HB][NP][8], o[HB][NP][8], m[HB], l[HB];
#pragma unroll
    for (int i = 0; i < HB; i++) {
        m[i] = -INFINITY, l[i] = 0.f;
#pragma unroll
        for (int j = 0; j < NP; j++)
#pragma unroll
            for (int e = 0; e < 8; e++) {
                q[i][j][e] = i < nh && l16 + 16 * j < nk ? sq[i * a.dnp + (l16 + 16 * j) * 8 + e] : 0.f;
                o[i][j][e] = 0.f;
            }
    }
    for (int kb = k0 + rg; kb < k1; kb += 16 * U) {
#pragma unroll
        for (int u = 0; u < U; u++) {
            const int k = kb + 16 * u;
            float c[NP][8], v[NP][8];
#pragma unroll
            for (int j = 0; j < NP; j++)
#pragma unroll
                for (int e = 0; e < 8; e++) c[j][e] = fh_up(nx[u][j].v[e]), v[j][e] = fh_up(ny[u][j].v[e]);
            fetch(k + 16 * U, nx[u], ny[u]);
            if (k >= k1) continue; // the same for the 16 lanes of a row
            if (k == mine)
#pragma unroll
                for (int j = 0; j < NP; j++)
#pragma unroll
                    for (int e = 0; e < 8; e++) {
                        c[j][e] = l16 + 16 * j < nk ? sk[(l16 + 16 * j) * 8 + e] : 0.f;
                        v[j][e] = l16 + 16 * j < nv ? sv[(l16 + 16 * j) * 8 + e] : 0.f;
                    }
#pragma unroll
            for (int i = 0; i < HB; i++) {
                float d = 0.f;
#pragma unroll
                for (int j = 0; j < NP; j++)
#pragma unroll
                    for (int e = 0; e < 8; e++) d = fmaf(q[i][j][e], c[j][e], d);
                d = fh_row16_sum(d);
                const float mn = fmaxf(m[i], d), r = exp2f(m[i] - mn), w = exp2f(d - mn);
                l[i] = l[i] * r + w;
                m[i] = mn;
#pragma unroll
                for (int j = 0; j < NP; j++)
#pragma unroll
                    for (int e = 0; e < 8; e++) o[i][j][e] = fmaf(w, v[j][e], o[i][j][e] * r);
            }
        }
    }
    // the four row groups of a wavefront, then the four wavefronts through the LDS
    const int sz = a.dvp + 2;
#pragma unroll
    for (int i = 0; i < HB; i++) {
        float mm = fmaxf(m[i], __shfl_xor(m[i], 16, 64));
        mm = fmaxf(mm, __shfl_xor(mm, 32, 64));
        const float f = m[i] == -INFINITY ? 0.f : exp2f(m[i] - mm);
        float ll = l[i] * f;
        ll += __shfl_xor(ll, 16, 64);
        ll += __shfl_xor(ll, 32, 64);
        float *dst = od + (wave * HB + i) * sz;
#pragma unroll
        for (int j = 0; j < NP; j++)
#pragma unroll
            for (int e = 0; e < 8; e++) {
                float x = o[i][j][e] * f;
                x += __shfl_xor(x, 16, 64);
                x += __shfl_xor(x, 32, 64);
                if (lane < 16 && l16 + 16 * j < nv) dst[(l16 + 16 * j) * 8 + e] = x;
            }
        if (lane == 0) dst[a.dvp] = mm, dst[a.dvp + 1] = ll;
    }
    __syncthreads();
    for (int i = 0; i < nh; i++) {
        float mm = -INFINITY, f[4], ll = 0.f;
#pragma unroll
        for (int w = 0; w < 4; w++) mm = fmaxf(mm, od[(w * HB + i) * sz + a.dvp]);
#pragma unroll
        for (int w = 0; w < 4; w++) {
            const float mw = od[(w * HB + i) * sz + a.dvp];
            f[w] = mw == -INFINITY ? 0.f : exp2f(mw - mm);
            ll += f[w] * od[(w * HB + i) * sz + a.dvp + 1];
        }
        float *dst = part + ((int64_t)(h0 + i) * splits + split) * sz;
        for (int x = tid; x < a.dvp; x += 256) {
            float v = 0.f;
#pragma unroll
            for (int w = 0; w < 4; w++) v = fmaf(f[w], od[(w * HB + i) * sz + x], v);
            dst[x] = v;
        }
        if (tid == 0) dst[a.dvp] = mm, dst[a.dvp + 1] = ll;
    }
}

// Merge of a head's parts by one wavefront: o [vdim] times out_scale.
__device__ __forceinline__ void fh_gqa_merge(const FhGqa &a, const float *part, int splits, int h, float *o) {
    static_assert(FH_GQA_MAX_SPLITS <= 64, "one part per lane");
    const float LOG2E = 1.4426950408889634f;
    const int lane = threadIdx.x & 63, sz = a.dvp + 2;
    const float *p = part + (int64_t)h * splits * sz;
    const float z = a.sink ? a.sink[h] * LOG2E : -INFINITY;
    const float m = lane < splits ? p[lane * sz + a.dvp] : -INFINITY, l = lane < splits ? p[lane * sz + a.dvp + 1] : 0.f;
    float mm = fmaxf(m, z);
#pragma unroll
    for (int i = 32; i > 0; i >>= 1) mm = fmaxf(mm, __shfl_xor(mm, i, 64));
    const float f = m == -INFINITY ? 0.f : exp2f(m - mm);
    float d = fh_wave_sum(f * l);
    if (a.sink) d += exp2f(z - mm);
    const float w = f / d * a.out_scale;
    for (int x0 = 0; x0 < a.vdim; x0 += 64) {
        const int x = x0 + lane < a.vdim ? x0 + lane : a.vdim - 1;
        float v = 0.f;
        for (int i0 = 0; i0 < splits; i0 += 8) { // eight requests on their way; parts behind the last one have the weight zero
            float y[8];
#pragma unroll
            for (int i = 0; i < 8; i++) y[i] = p[(i0 + i < splits ? i0 + i : splits - 1) * sz + x];
#pragma unroll
            for (int i = 0; i < 8; i++) v = fmaf(__shfl(w, i0 + i, 64), y[i], v);
        }
        if (x0 + lane < a.vdim) o[x] = v;
    }
}
#endif
