// Device helpers and host launchers for dense bf16 weights (FH_BF16) with bf16 or f32 activations: the products of the
// layer-list decoders (fh_hybrid.hip).  Weight rows are row-major with a stride of k rounded up to 64 elements, the
// rows are rounded up to 16, and all padding is zero; activation rows use the same stride, so no kernel has an edge
// along k.
#pragma once
#include "fh_internal.h"

typedef __bf16 fh_bf;
typedef __bf16 fh_bf8 __attribute__((ext_vector_type(8)));
typedef __bf16 fh_bf4 __attribute__((ext_vector_type(4)));
typedef float fh_f4 __attribute__((ext_vector_type(4)));
struct fh_f8 { float v[8]; };

static inline int64_t fh_pad64(int64_t k) { return (k + 63) / 64 * 64; }

__device__ __forceinline__ float fh_bf_f32(uint16_t b) { return __uint_as_float((uint32_t)b << 16); }
__device__ __forceinline__ uint16_t fh_f32_bf(float f) {
    const fh_bf b = (fh_bf)f;
    uint16_t u;
    __builtin_memcpy(&u, &b, 2);
    return u;
}
// low / high half of a 32-bit word of two bf16
__device__ __forceinline__ float fh_bf_lo(uint32_t w) { return __uint_as_float(w << 16); }
__device__ __forceinline__ float fh_bf_hi(uint32_t w) { return __uint_as_float(w & 0xFFFF0000u); }

template <typename T> __device__ __forceinline__ T fh_to(float f);
template <> __device__ __forceinline__ float fh_to<float>(float f) { return f; }
template <> __device__ __forceinline__ uint16_t fh_to<uint16_t>(float f) { return fh_f32_bf(f); }
__device__ __forceinline__ float fh_up(float f) { return f; }
__device__ __forceinline__ float fh_up(uint16_t b) { return fh_bf_f32(b); }

__device__ __forceinline__ float fh_wave_sum(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
    return v;
}
// silu, softplus and the logistic function with the full-precision exponential
__device__ __forceinline__ float fh_silu_f(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float fh_softplus_f(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float fh_sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }

// Eight k-values of an MFMA operand in the layout of v_mfma_f32_16x16x32_bf16 (lane l: row l % 16, k = 8 (l / 16) .. + 7)
// and one 16 x 16 x 32 step on them.  f32 operands keep the same layout: eight v_mfma_f32_16x16x4_f32, each with one of
// the lane's values, add up to the same 32 of k in true f32.
template <typename T> struct FhFrag;
template <> struct FhFrag<uint16_t> { typedef fh_bf8 type; };
template <> struct FhFrag<float> { typedef fh_f8 type; };
__device__ __forceinline__ void fh_frag_load(fh_bf8 &f, const uint16_t *p) {
    const uint4 r = *(const uint4 *)p;
    __builtin_memcpy(&f, &r, 16);
}
__device__ __forceinline__ void fh_frag_load(fh_f8 &f, const float *p) {
    const float4 a = *(const float4 *)p, b = *(const float4 *)(p + 4);
    f.v[0] = a.x, f.v[1] = a.y, f.v[2] = a.z, f.v[3] = a.w;
    f.v[4] = b.x, f.v[5] = b.y, f.v[6] = b.z, f.v[7] = b.w;
}
__device__ __forceinline__ fh_f4 fh_mma32(const fh_bf8 &a, const fh_bf8 &b, fh_f4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ fh_f4 fh_mma32(const fh_f8 &a, const fh_f8 &b, fh_f4 c) {
#pragma unroll
    for (int e = 0; e < 8; e++) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.v[e], b.v[e], c, 0, 0, 0);
    return c;
}

// ---------------------------------------------------------------- host launchers
// Storage of activations between kernels: FH_F32, or FH_BF16_ACT for decoders that serve in bf16.
enum { FH_BF16_ACT = 2 };
static inline size_t fh_act_size(int dtype) { return dtype == FH_BF16_ACT ? 2 : 4; }

// Row groups of a grouped product: tile i covers rows [row0, row0 + rows) that all belong to group `group`.
struct FhTile { int group, row0, rows, pad; };

enum {
    FH_GEMM_F32 = 0,        // y f32 [m, ldy]
    FH_GEMM_ACT = 1,        // y in the activation type [m, ldy]
    FH_GEMM_ACT_T = 2,      // y in the activation type, transposed: [n, ldy], ldy >= m
    FH_GEMM_SWIGLU = 3,     // weight rows in alternating groups of 16 (gate, up): y = silu(gate) * up, activation type [m, ldy]
    FH_GEMM_RELU2 = 4       // y = max(x, 0)^2, activation type [m, ldy]
};
struct FhGemm {
    const uint16_t *w = nullptr; // [n, kp]
    int64_t w_group = 0;         // elements between the weights of two groups
    const void *x = nullptr;     // [rows, kp]
    const int *gather = nullptr; // row of x behind row i (NULL: i)
    void *y = nullptr;
    int64_t ldy = 0;
    int n = 0, kp = 0, m = 0;    // n: weight rows of a group
    const FhTile *tiles = nullptr; // grouped: device table and its fill count
    const int *n_tiles = nullptr;
    int max_tiles = 0, tile_rows = 64; // rows an entry may cover: 64, or 128 with bf16 activations
};
fh_status fh_gemm(fh_device *dev, int dtype, int epi, const FhGemm &g);

// y[seg][row] = W_seg[row, :] . n(x), n(x) = x / rms(x) * w (w NULL: x as it is).  norm_out (optional) receives n(x).
struct FhMvSeg { const uint16_t *w; float *y; int n; };
fh_status fh_matvec_norm(fh_device *dev, const float *x, int k, const float *w, float eps, const FhMvSeg *segs, int n_segs,
                         float *norm_out);
// f32 rows -> activation rows of stride kp: plain copy, or RMS norm with weight w (w NULL: copy)
fh_status fh_rows_to_act(fh_device *dev, int dtype, const float *x, int64_t ldx, int rows, int k, const float *w, float eps,
                         void *y, int kp);

// The row table of a product whose `groups` groups have s rows each, group after group (FhGemm::tiles, n_tiles).
static inline int fh_group_tile_rows(const fh_device *dev, int dtype, int groups, int s, int n) {
    return dtype != FH_F32 && (int64_t)groups * ((s + 127) / 128) * ((n + 127) / 128) >= dev->compute_units ? 128 : 64;
}
fh_status fh_group_tiles(fh_device *dev, int groups, int s, int tile_rows, FhTile *tiles, int *n_tiles);

// ---------------------------------------------------------------- residual streams that are normed at a sublayer's end
// x_out = x + y / rms(y) * w per row, and (act not NULL) x_out as activation rows of stride kp; x_out may be x.
fh_status fh_add_normed(fh_device *dev, int dtype, const float *x, const float *y, int rows, int k, const float *w, float eps,
                        float *x_out, void *act, int kp);
// x[t] = table row ids[t] + pos row (pos + t, or *pos_dev for one token); pos_table NULL: without.  Also activation rows.
fh_status fh_embed_at(fh_device *dev, int dtype, const fh_qmatrix *table, const fh_qmatrix *pos_table, const uint32_t *ids, int s,
                      int pos, const int *pos_dev, float *x, void *act, int kp);

// Token shift: mixture n of token t is x_t + (x_(t-1) - x_t) * mu_n.  The row ahead of the portion is kept in a state of two
// rows (position p in row p % 2; nothing is read at position 0).
enum { FH_SHIFT_MAX = 6 };
struct FhShift {
    int n = 0;
    const float *mu[FH_SHIFT_MAX] = {};
    void *y[FH_SHIFT_MAX] = {};   // [s, kp]
    int f32[FH_SHIFT_MAX] = {};   // rows in f32 whatever the activation type
};
// y = tanh(W x) in 32 bits, W [n, kp] for a small n: x [rows, kp] f32, y [rows, ldy] f32 with zeros from n on.
fh_status fh_low_rank_tanh(fh_device *dev, const float *x, int kp, int rows, const uint16_t *w, int n, float *y, int ldy);
fh_status fh_token_shift(fh_device *dev, int dtype, const FhShift &m, const float *x, int s, int k, int pos, float *state, int kp);

// Decode: x' = x + y / rms(y) * w (y NULL: x), then up to FH_MV_MAX matrices on mixtures of x' (mu NULL: x' itself).  One
// workgroup stores x' (x_out, not x) and, with a state, the row of this position.
// With a gate: x' = x / rms(x) * w * silu(gate) * scale, the norm over `groups` equal groups of x (w NULL: without).
enum { FH_MV_ACT_NONE = 0, FH_MV_ACT_RELU2 = 1, FH_MV_ACT_TANH = 2, FH_MV_MAX = 6 };
struct FhMvMix { const uint16_t *w; const float *mu; float *y; int n, act; };
struct FhMvAdd {
    const float *x = nullptr, *y = nullptr, *w = nullptr;
    float eps = 0.f;
    float *x_out = nullptr;
    float *state = nullptr;       // [2][k]
    const int *pos_dev = nullptr;
    const float *gate = nullptr;
    int groups = 0, w_len = 0;
    float scale = 1.f;
};
fh_status fh_matvec_mix(fh_device *dev, const FhMvAdd &in, int k, const FhMvMix *segs, int n_segs);

#ifdef __HIPCC__
// Dimension i of a head after rotation: pairs (2i, 2i + 1), or (i, i + pairs) with `halves`, of the first 2 pairs dimensions;
// at(i) gives dimension i before it, ct / st the row of the position.
template <typename F>
__device__ __forceinline__ float fh_rotated(F at, int i, int pairs, int halves, const float *ct, const float *st) {
    const float v = at(i);
    if (i >= 2 * pairs) return v;
    if (halves) return i < pairs ? v * ct[i] - at(i + pairs) * st[i] : v * ct[i - pairs] + at(i - pairs) * st[i - pairs];
    const int p = i >> 1;
    return i & 1 ? v * ct[p] + at(i - 1) * st[p] : v * ct[p] - at(i + 1) * st[p];
}
#endif
