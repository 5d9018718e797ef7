// Mixture-of-experts feed-forward: softmax router, the `top` best experts of a token weighted by scale times their score,
// and optionally one more expert that is always on.  Expert weights are stacked: gate | up rows in
// alternating groups of 16, [experts][2 ffp][kp], and down [experts][dp][ffp], with ffp = ff rounded up to 64 (zero rows)
// and dp = the width rounded up to 16.
#pragma once
#include "fh_dense.h"

enum { FH_MOE_MAX_EXPERTS = 1024 };
struct FhMoe {
    int experts = 0, top = 0, ff = 0, ffp = 0;   // experts 0: no routed part
    float scale = 1.f;
    int col_z = 0;                               // router logits in a projection row
    const uint16_t *gate_up = nullptr, *down = nullptr;
    int64_t gu_stride = 0, down_stride = 0;      // elements per expert
    int sff = 0, sffp = 0;                       // the always-on expert (0: none)
    const uint16_t *s_gate_up = nullptr, *s_down = nullptr;
};
// Work arrays of a prefill portion.
struct FhMoeWork {
    int *ids;       // [t, top] chosen experts
    float *wts;     // [t, top]
    int *src;       // [t * top] token behind a sorted assignment
    int *inv;       // [t, top] sorted place of an assignment
    FhTile *tiles;  // fh_moe_max_tiles
    int *n_tiles;
    void *act;      // [t * top, ffp] activation rows
    float *y;       // [t * top, width]
    void *s_act;    // [t, sffp]
    float *s_y;     // [t, width]
};
// rows per tile: the larger ones where an expert has rows to fill them on average
static inline int fh_moe_tile_rows(const FhMoe &m, int dtype, int s) {
    return dtype != FH_F32 && (int64_t)s * m.top >= (int64_t)m.experts * 96 ? 128 : 64;
}
static inline int fh_moe_max_tiles(const FhMoe &m, int s, int tile_rows) { return s * m.top / tile_rows + m.experts; }
// x [s, width] += mix [s, width] + the feed-forward of the activation rows h [s, kp]
fh_status fh_moe_prefill(fh_device *dev, int dtype, const FhMoe &m, const void *h, int kp, const float *proj, int64_t ldp,
                         int s, int width, const FhMoeWork &w, const float *mix, float *x);

#ifdef __HIPCC__
// The n-th best expert of one token and its weight, for all n < count, by one wavefront: every lane keeps the logits
// e = lane + 64 i.  Ties go to the smaller index.  pick(n, expert, weight) runs in every lane.
template <typename F>
__device__ __forceinline__ void fh_moe_route(const float *z, int experts, float scale, int count, F pick) {
    const int lane = threadIdx.x & 63;
    float v[FH_MOE_MAX_EXPERTS / 64];
    const int per = (experts + 63) / 64;
    float mx = -INFINITY;
#pragma unroll
    for (int i = 0; i < FH_MOE_MAX_EXPERTS / 64; i++) {
        v[i] = i < per && lane + 64 * i < experts ? z[lane + 64 * i] : -INFINITY;
        mx = fmaxf(mx, v[i]);
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o, 64));
    float den = 0.f;
#pragma unroll
    for (int i = 0; i < FH_MOE_MAX_EXPERTS / 64; i++) den += v[i] == -INFINITY ? 0.f : expf(v[i] - mx);
    den = fh_wave_sum(den);
    for (int n = 0; n < count; n++) {
        float best = -INFINITY;
        int bi = 0x7FFFFFFF;
#pragma unroll
        for (int i = 0; i < FH_MOE_MAX_EXPERTS / 64; i++)
            if (v[i] > best) best = v[i], bi = lane + 64 * i;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) {
            const float ob = __shfl_xor(best, o, 64);
            const int oi = __shfl_xor(bi, o, 64);
            if (ob > best || (ob == best && oi < bi)) best = ob, bi = oi;
        }
        if (bi >= experts) bi = 0; // only when no logit is a number
        pick(n, bi, expf(best - mx) / den * scale);
#pragma unroll
        for (int i = 0; i < FH_MOE_MAX_EXPERTS / 64; i++)
            if (bi == lane + 64 * i) v[i] = -INFINITY;
    }
}
#endif
