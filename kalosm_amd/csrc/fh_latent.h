// Attention over a low-rank latent.  A position caches its RMS-normed latent vector c and a rotated key fragment kr that
// all heads use; the heads' keys and values are linear maps of c.
//   score(i, j) = (q_h . W_uk,h c_j + qr_h . kr_j) * scale,   out_h = W_uv,h sum_j p_ij c_j
// Prefill expands keys and values of the visible positions and runs a tiled attention over them; a decode step moves
// W_uk to the query and W_uv behind the sum, so that it reads the cached rows only.
// With a window w, key j is visible to query i while 0 <= i - j < w; a sink adds exp(sink_h) to a head's denominator.
// Scores, weights and sums are f32; in bf16 serving the operands of the prefill products are bf16, the weights p of the
// second product as two terms (hi + lo).
//
// Cache rows (fh_kvcache of one layer, no V plane, a ring of at most `window` rows): [c: r8 | rotated key: drp], both
// padded with zeros to multiples of 8.
#pragma once
#include "fh_recurrent.h"
#include "fh_window_attn.h"

struct FhLatent {
    int heads = 0, dn = 0, dr = 0, dv = 0, rank = 0;
    int dnp = 0, drp = 0, r8 = 0, rp = 0;    // dn, dr, rank rounded up to 8, rank rounded up to 64
    int col_q = 0, col_kv = 0;               // columns of a projection row: [heads][dn | dr], [rank | dr]
    int window = 0;                          // 0: all earlier positions
    float scale = 1.f, eps = 0.f;
    const float *c_norm = nullptr, *sink = nullptr; // [rank], [heads] or NULL
    const float *cos_t = nullptr, *sin_t = nullptr; // [positions, pairs]
    int pairs = 0;                           // rotated pairs of the dr dimensions
    const uint16_t *uk = nullptr;            // [heads * dnp, rp]
    const uint16_t *uv = nullptr;            // [heads * dv, rp]
};
static inline int fh_latent_row(const FhLatent &a) { return a.r8 + a.drp; }

// Work arrays of a prefill portion over `keys` = old + new positions.
struct FhLatentWork {
    void *lat, *kr;   // [keys, rp], [keys, drp]
    void *kn, *vt;    // [keys, heads * dnp], [heads * dv, ldt]
    void *q;          // [s, heads, dq]
    int64_t ldt;
};
int fh_latent_dq(const FhLatent &a); // padded query / key length of the attention kernel, 0: unsupported
// keys of a portion of s tokens at position pos: those before it that its first token still sees, and its own
static inline int fh_latent_old(const FhLatent &a, int pos) { return a.window && a.window - 1 < pos ? a.window - 1 : pos; }
fh_status fh_latent_prefill(fh_device *dev, int dtype, const FhLatent &a, fh_kvcache *cache, const float *proj, int64_t ldp,
                            int s, int pos, const FhLatentWork &w, void *o, int kp);

enum { FH_LATENT_MAX_SPLITS = 64 };
static inline size_t fh_latent_part_floats(const FhLatent &a) { return (size_t)a.heads * FH_LATENT_MAX_SPLITS * (a.r8 + 2); }
// Decode step behind the absorbed queries qa [heads, fh_latent_row] (scaled to base-2 exponents): o [heads * dv]
fh_status fh_latent_decode(fh_device *dev, int dtype, const FhLatent &a, const fh_kvcache *cache, const int *pos_dev,
                           const float *qa, float *part, float *o);
