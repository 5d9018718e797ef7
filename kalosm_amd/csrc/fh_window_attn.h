// Prefill attention over the keys and values of a portion's visible positions, laid out row by row: grouped heads, a sliding
// window, the first `keep` positions always visible, a learned sink per head.
//   query i (position pos + i) sees row j of position p when p <= pos + i and (pos + i - p < window or p < keep)
// Rows 0 .. kept - 1 hold the positions of their number, row j >= kept holds position j + gap (what a long sequence has
// between the kept tokens and the window has no rows).  Scores, weights and sums are f32; with bf16 operands a weight is
// multiplied as two terms (hi + lo).
#pragma once
#include "fh_dense.h"

struct FhWindowAttn {
    int heads = 0, rep = 1;          // query heads, query heads per key head
    int dnp = 0, drp = 0, dv = 0;    // per-head and shared part of a key (multiples of 8), value length
    int window = 0, keep = 0;        // window 0: all earlier positions
    int pos = 0, kept = 0, gap = 0;
    float scale = 1.f, out_scale = 1.f;
    const float *sink = nullptr;     // [heads] or NULL
};
int fh_window_dq(int dims); // padded query / key length of the kernel, 0: unsupported
// q [s, heads, fh_window_dq], kn [keys, heads / rep, dnp], kr [keys, drp] (all heads), vt [heads / rep * dv, ldt];
// o rows of stride ldo: heads * dv values, zeros up to kp.
fh_status fh_window_attn(fh_device *dev, int dtype, const FhWindowAttn &a, const void *q, const void *kn, const void *kr,
                         const void *vt, int64_t ldt, int s, int keys, void *o, int ldo, int kp);

// ---------------------------------------------------------------- device parts: pieces of eight elements
template <typename T> struct FhPiece { T v[8]; };
template <typename T>
__device__ __forceinline__ FhPiece<T> fh_zero_piece() {
    FhPiece<T> p;
#pragma unroll
    for (int e = 0; e < 8; e++) p.v[e] = 0;
    return p;
}
template <typename T>
__device__ __forceinline__ FhPiece<T> fh_ld_piece(const T *p) {
    FhPiece<T> r;
    struct alignas(16) A { T v[8]; };
    const A a = *(const A *)p;
    __builtin_memcpy(&r, &a, sizeof r);
    return r;
}
template <typename T>
__device__ __forceinline__ void fh_st_piece(T *p, const FhPiece<T> &r) {
    struct alignas(16) A { T v[8]; };
    A a;
    __builtin_memcpy(&a, &r, sizeof r);
    *(A *)p = a;
}
