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
    const int wide = a.dnp > 128 || a.dvp > 128 ? 256 : 128, parts = 4 * FH_GQA_HEADS * (a.dvp + 4), tmp = FH_GQA_HEADS * wide;
    return (size_t)((FH_GQA_HEADS + 2) * wide + (parts > tmp ? parts : tmp)) * 4;
}

#ifdef __HIPCC__
#include "fh_mv_lanes.h"
#include "fh_recurrent.h"
// One head of at most 64 J values in a wavefront's registers: value, norm weight, and the cosine and sine of its pair.  The
// request and the work are apart, so that several heads' requests can be on their way at once; no request is conditional.
template <int J> struct FhHead { float x[J], w[J], c[J], s[J]; };
template <int J>
__device__ __forceinline__ void fh_head_load(const FhGqa &a, const float *raw, const float *w, const float *ct, const float *st, FhHead<J> &h) {
    const int lane = threadIdx.x & 63;
#pragma unroll
    for (int j = 0; j < J; j++) {
        const int i = lane + 64 * j, ic = i < a.dim ? i : a.dim - 1;
        int p = a.halves ? i < a.pairs ? i : i - a.pairs : i >> 1;
        p = p < a.pairs ? p : a.pairs - 1;
        h.x[j] = raw[ic];
        h.w[j] = w ? w[ic] : 1.f;
        h.c[j] = ct[p];
        h.s[j] = st[p];
    }
#pragma unroll
    for (int j = 0; j < J; j++) {
        const int i = lane + 64 * j;
        h.x[j] = i < a.dim ? h.x[j] : 0.f;
        h.c[j] = i < 2 * a.pairs ? h.c[j] : 1.f;
        h.s[j] = i < 2 * a.pairs ? h.s[j] : 0.f;
    }
}
// RMS norm (norm 0: none) and rotation: dst [64 J] times mul with zeros from dim on, through `tmp` [64 J] (LDS).
template <int J>
__device__ __forceinline__ void fh_head_rotate(const FhGqa &a, FhHead<J> &h, int norm, float mul, float *tmp, float *dst) {
    const int lane = threadIdx.x & 63;
    if (norm) {
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < J; j++) ss = fmaf(h.x[j], h.x[j], ss);
        ss = rows_sum(fh_row16_sum(ss));
        const float inv = 1.0f / sqrtf(ss / (float)a.dim + a.eps);
#pragma unroll
        for (int j = 0; j < J; j++) h.x[j] *= inv * h.w[j];
    }
#pragma unroll
    for (int j = 0; j < J; j++) tmp[lane + 64 * j] = h.x[j];
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
#pragma unroll
    for (int j = 0; j < J; j++) {
        const int i = lane + 64 * j;
        const bool second = a.halves ? i >= a.pairs : i & 1;
        int o = a.halves ? second ? i - a.pairs : i + a.pairs : i ^ 1;
        o = o < 64 * J ? o : i; // not turned there
        const float v = tmp[o] * h.s[j];
        dst[i] = (h.x[j] * h.c[j] + (second ? v : -v)) * mul;
    }
}

__device__ __forceinline__ float fh_rows_max(float v) { // maximum over the four rows of 16 lanes, in every row
    const uint32_t u = __float_as_uint(v);
    auto s16 = __builtin_amdgcn_permlane16_swap(u, u, false, false);
    v = fmaxf(__uint_as_float(s16[0]), __uint_as_float(s16[1]));
    const uint32_t w = __float_as_uint(v);
    auto s32 = __builtin_amdgcn_permlane32_swap(w, w, false, false);
    return fmaxf(__uint_as_float(s32[0]), __uint_as_float(s32[1]));
}

// Workgroup b of fh_gqa_blocks: up to FH_GQA_HEADS query heads of one key head against one part of the cache.  The 16 lanes
// of a DPP row take U cached rows at a time, pieces of 8 elements, NP pieces per lane (dim and vdim at most 128 NP).  Lengths
// are padded with zeros in the query, so that nothing in the loop is conditional.  The row of this position is computed here,
// used from the LDS and stored by one of the workgroups that need it.
template <typename T, int NP>
__device__ __forceinline__ void fh_gqa_step(const FhGqa &a, const float *proj, T *ring, int cap, int pos, int splits, int b,
                                            float *__restrict__ part, float *lds) {
    constexpr int HB = FH_GQA_HEADS, U = NP == 1 ? 4 : 2, W = 128 * NP, J = 2 * NP;
    const float LOG2E = 1.4426950408889634f;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, l16 = lane & 15, rg = tid >> 4;
    const int rep = a.heads / a.kv_heads, groups = (rep + HB - 1) / HB, hg = b % groups, bb = b / groups;
    const int split = bb % splits, kh = bb / splits, h0 = kh * rep + hg * HB, nh = rep - hg * HB < HB ? rep - hg * HB : HB;
    const int n = pos + 1 < cap ? pos + 1 : cap, mine = fh_ring_row(pos, cap, a.keep);
    const int per = ((n + splits - 1) / splits + 15) / 16 * 16;
    const int k0 = split * per, k1 = k0 + per < n ? k0 + per : n;
    const int row = a.kv_heads * (a.dnp + a.dvp), nk = a.dnp / 8, nv = a.dvp / 8;
    const bool own = mine >= k0 && mine < k1;
    float *sq = lds, *sk = sq + HB * W, *sv = sk + W, *od = sv + W;
    const T *kp_[NP], *vp_[NP];
#pragma unroll
    for (int i = 0; i < NP; i++) { // pieces behind a row's end read another one, against zeros of the query or for nothing
        kp_[i] = ring + kh * a.dnp + (l16 + 16 * i < nk ? l16 + 16 * i : 0) * 8;
        vp_[i] = ring + a.kv_heads * a.dnp + kh * a.dvp + (l16 + 16 * i < nv ? l16 + 16 * i : 0) * 8;
    }
    FhPiece<T> nx[U][NP], ny[U][NP];
    // rows behind the part's end read the lane group's first row instead
    auto at = [&](int kb, int u) { return kb + 16 * u < k1 ? kb + 16 * u : kb < k1 ? kb : 0; };
    auto fetch = [&](int kb) {
#pragma unroll
        for (int u = 0; u < U; u++)
#pragma unroll
            for (int i = 0; i < NP; i++) {
                nx[u][i] = fh_ld_piece(kp_[i] + (int64_t)at(kb, u) * row);
                ny[u][i] = fh_ld_piece(vp_[i] + (int64_t)at(kb, u) * row);
            }
    };
    fetch(k0 + rg); // before the query is worked on
    const float *ct = a.cos_t + (int64_t)pos * a.pairs, *st = a.sin_t + (int64_t)pos * a.pairs;
    FhHead<J> hq, hk;
    fh_head_load<J>(a, proj + a.col_q + (h0 + (wave < nh ? wave : 0)) * a.dim, a.q_norm, ct, st, hq);
    float hv = proj[a.col_v + kh * a.vdim + (tid < a.vdim ? tid : 0)];
    if (own && wave == 0) fh_head_load<J>(a, proj + a.col_k + kh * a.dim, a.k_norm, ct, st, hk);
    fh_head_rotate<J>(a, hq, a.q_norm != nullptr, a.scale * LOG2E, od + wave * W, sq + wave * W);
    if (own) {
        if (wave == 0) fh_head_rotate<J>(a, hk, a.k_norm != nullptr, 1.f, od, sk);
        hv = tid < a.vdim ? fh_up(fh_to<T>(hv)) : 0.f; // as the cache holds it
        if (tid < W) sv[tid] = hv;
    }
    __syncthreads();
    if (own) {
        if (tid < W) {
            const T kt = fh_to<T>(sk[tid]);
            sk[tid] = fh_up(kt);
            if (hg == 0) {
                T *dst = ring + (int64_t)mine * row;
                if (tid < a.dnp) dst[kh * a.dnp + tid] = kt;
                if (tid < a.dvp) dst[a.kv_heads * a.dnp + kh * a.dvp + tid] = fh_to<T>(hv);
            }
        }
        __syncthreads();
    }
    float q[HB][NP][8], o[HB][NP][8], m[HB], l[HB];
#pragma unroll
    for (int i = 0; i < HB; i++) {
        m[i] = -INFINITY, l[i] = 0.f;
#pragma unroll
        for (int j = 0; j < NP; j++) {
            __builtin_memcpy(q[i][j], sq + i * W + (l16 + 16 * j) * 8, 32);
#pragma unroll
            for (int e = 0; e < 8; e++) o[i][j][e] = 0.f;
        }
    }
    for (int kb = k0 + rg; kb < k1; kb += 16 * U) {
        float c[U][NP][8], v[U][NP][8], d[U][HB];
#pragma unroll
        for (int u = 0; u < U; u++) {
#pragma unroll
            for (int j = 0; j < NP; j++)
#pragma unroll
                for (int e = 0; e < 8; e++) c[u][j][e] = fh_up(nx[u][j].v[e]), v[u][j][e] = fh_up(ny[u][j].v[e]);
            if (at(kb, u) == mine)
#pragma unroll
                for (int j = 0; j < NP; j++) {
                    __builtin_memcpy(c[u][j], sk + (l16 + 16 * j) * 8, 32);
                    __builtin_memcpy(v[u][j], sv + (l16 + 16 * j) * 8, 32);
                }
        }
        fetch(kb + 16 * U);
#pragma unroll
        for (int u = 0; u < U; u++)
#pragma unroll
            for (int i = 0; i < HB; i++) {
                float x = 0.f;
#pragma unroll
                for (int j = 0; j < NP; j++)
#pragma unroll
                    for (int e = 0; e < 8; e++) x = fmaf(q[i][j][e], c[u][j][e], x);
                x = fh_row16_sum(x);
                d[u][i] = kb + 16 * u < k1 ? x : -INFINITY;
            }
#pragma unroll
        for (int i = 0; i < HB; i++) { // the first of the rows is there, so the maximum is a number
            float mn = m[i];
#pragma unroll
            for (int u = 0; u < U; u++) mn = fmaxf(mn, d[u][i]);
            const float r = __builtin_amdgcn_exp2f(m[i] - mn);
            m[i] = mn, l[i] *= r;
#pragma unroll
            for (int j = 0; j < NP; j++)
#pragma unroll
                for (int e = 0; e < 8; e++) o[i][j][e] *= r;
#pragma unroll
            for (int u = 0; u < U; u++) {
                const float w = __builtin_amdgcn_exp2f(d[u][i] - mn);
                l[i] += w;
#pragma unroll
                for (int j = 0; j < NP; j++)
#pragma unroll
                    for (int e = 0; e < 8; e++) o[i][j][e] = fmaf(w, v[u][j][e], o[i][j][e]);
            }
        }
    }
    // the four row groups of a wavefront, then the four wavefronts through the LDS
    const int sz = a.dvp + 2, ls = a.dvp + 4;
#pragma unroll
    for (int i = 0; i < HB; i++) {
        const float mm = fh_rows_max(m[i]), f = m[i] == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m[i] - mm), ll = rows_sum(l[i] * f);
        float *dst = od + (wave * HB + i) * ls;
#pragma unroll
        for (int j = 0; j < NP; j++) {
            float x[8];
#pragma unroll
            for (int e = 0; e < 8; e++) x[e] = rows_sum(o[i][j][e] * f);
            if (lane < 16 && l16 + 16 * j < nv) __builtin_memcpy(dst + (l16 + 16 * j) * 8, x, 32);
        }
        if (lane == 0) dst[a.dvp] = mm, dst[a.dvp + 1] = ll;
    }
    __syncthreads();
    const int x = tid % W;
#pragma unroll
    for (int i0 = 0; i0 < HB; i0 += 256 / W) {
        const int i = i0 + tid / W;
        if (i >= nh) break;
        float mw[4], mm = -INFINITY, ll = 0.f, v = 0.f;
#pragma unroll
        for (int w = 0; w < 4; w++) mw[w] = od[(w * HB + i) * ls + a.dvp], mm = fmaxf(mm, mw[w]);
#pragma unroll
        for (int w = 0; w < 4; w++) {
            const float f = mw[w] == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(mw[w] - mm);
            ll += f * od[(w * HB + i) * ls + a.dvp + 1];
            v = fmaf(f, od[(w * HB + i) * ls + (x < a.dvp ? x : 0)], v);
        }
        float *dst = part + ((int64_t)(h0 + i) * splits + split) * sz;
        if (x < a.dvp) dst[x] = v;
        if (x == 0) dst[a.dvp] = mm, dst[a.dvp + 1] = ll;
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
