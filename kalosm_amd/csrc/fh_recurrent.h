// Linear recurrences with a matrix state per head, in one form:
//   S_t = G_t S_(t-1) + k_t u_t^T,   o_t = S_t^T q_t [+ D v_t]
//   gated delta rule:  G = exp(la_t), u_t = beta_t (v_t - (exp(la_t) S_(t-1))^T k_t), q and k unit vectors, q scaled
//   state space:       G = exp(la_t), u_t = beta_t v_t  (beta the step size, k / q / v its B / C / x)
//   retention:         G a constant of the head, u_t = v_t, q and k rotated by their position, k scaled
//   channel decay:     G = diag(exp(la_t)), one la per key channel, u_t = v_t, and the output reads the state before the
//                      token's own contribution joins it, which counts with a learned bonus per channel instead:
//                      o_t = (S_(t-1) + diag(bonus) k_t v_t^T)^T q_t
// Delta rule and state space: q, k and v pass a short causal convolution and silu; la = -exp(A_log) softplus(a + dt_bias).
// Channel decay: la = -exp(W_2 tanh(W_1 x) + w0).  All of it is f32.
// Per sequence and layer there are two pieces of state (FhRecState): S, one matrix per head stored column by column
// ([heads][vdim][dim]), and what the inputs need of earlier tokens: the projections of the last `taps` positions in a ring
// (position p in row p % taps), or the last two rows of a token shift.  Position 0 reads neither, so nothing is cleared
// between sequences.
#pragma once
#include "fh_dense.h"

enum { FH_REC_SPACE = 0, FH_REC_DELTA = 1, FH_REC_RETENTION = 2, FH_REC_CHANNEL = 3 };
struct FhRecurrent {
    int kind = FH_REC_SPACE;
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0, taps = 1;
    int col_q = 0, col_k = 0, col_v = 0, col_b = 0, col_a = 0, col_g = 0; // columns of a projection row
    const float *conv_q = nullptr, *conv_k = nullptr, *conv_v = nullptr;  // [channels, taps]
    const float *bias_q = nullptr, *bias_k = nullptr, *bias_v = nullptr;  // NULL: none
    const float *a_log = nullptr, *dt_bias = nullptr, *d_skip = nullptr;  // [heads]
    const float *norm = nullptr;                     // [norm_len], NULL: no weight
    int norm_len = 0, norm_groups = 0, gate_first = 0; // gate_first: silu(gate) before the norm instead of after it
    float eps = 0.f, q_scale = 1.f, k_scale = 1.f, out_scale = 1.f;
    // retention
    const float *log_decay = nullptr;                // [heads]
    const float *cos_t = nullptr, *sin_t = nullptr;  // [positions, pairs]
    int pairs = 0, halves = 0;                       // fh_rotated
    // channel decay
    const float *bonus = nullptr, *w0 = nullptr;     // [heads * dim]
    const uint16_t *w2 = nullptr;                    // [heads * dim, rp]
    int rank = 0, rp = 0;                            // low rank of the decay, rounded up to 64
    __host__ __device__ bool delta() const { return kind == FH_REC_DELTA; }
};
static inline int fh_rec_channels(const FhRecurrent &r) { return 2 * r.kv_heads * r.dim + r.heads * r.vdim; }
// rows of q and k in the work arrays of a portion: dim rounded up to a size the chunked form has, zeros in the padding
static inline int fh_rec_dp(const FhRecurrent &r) { return r.dim <= 32 ? 32 : r.dim <= 64 ? 64 : r.dim <= 128 ? 128 : 256; }
static inline int fh_rec_inner(const FhRecurrent &r) { return r.heads * r.vdim; }

// State of one recurrent layer of one sequence.
struct FhRecState {
    float *s = nullptr;    // [heads][vdim][dim]
    float *conv = nullptr; // [taps][channels]; channel decay: [2][width], the rows of the token shift
};

// Work arrays of a prefill portion, rows of one token each.
struct FhRecWork {
    float *q, *k;     // [t, kv_heads * fh_rec_dp]
    float *v;         // [t, heads * vdim]
    float *beta, *la; // [t, heads]
    float *o;         // [t, heads * vdim]
    float *chunk;     // scratch of the chunked form (fh_rec_chunk_floats)
};
size_t fh_rec_chunk_floats(const FhRecurrent &r, int s);
// One portion of s tokens at position pos: proj rows [s, ldp] -> normed, gated activation rows y [s, kp].
fh_status fh_recurrent_prefill(fh_device *dev, int dtype, const FhRecurrent &r, const FhRecState &st, const float *proj,
                               int64_t ldp, int s, int pos, const FhRecWork &w, void *y, int kp);
// The same for channel decay, whose inputs come from products of their own: q, k, v, gate [s, heads * dim] and the decays'
// argument z ahead of w0, all f32.  Output rows have the stride ldy, zeros from heads * dim up to kp.
struct FhRecRows { const float *q, *k, *v, *g, *z; };
fh_status fh_recurrent_channel(fh_device *dev, int dtype, const FhRecurrent &r, const FhRecState &st, const FhRecRows &in, int s, int pos,
                               const FhRecWork &w, void *y, int ldy, int kp);

// ---------------------------------------------------------------- device parts shared with the decode step
__device__ __forceinline__ float fh_row16_sum(float v) { // sum over the 16 lanes of a DPP row, in every lane
#define FH_ROR(N_) v += __uint_as_float(__builtin_amdgcn_update_dpp(0, __float_as_uint(v), 0x120 + N_, 0xF, 0xF, true))
    FH_ROR(8);
    FH_ROR(4);
    FH_ROR(2);
    FH_ROR(1);
#undef FH_ROR
    return v;
}

// Logarithm of a channel's decay.  A factor below e^-30 leaves nothing of a 32-bit state either way; the limit keeps sums of
// logarithms short.
__device__ __forceinline__ float fh_rec_la(float z) { return fmaxf(-expf(z), -30.f); }

// Convolution and silu of channel ch (q | k | v order) at position pos + t; projections of earlier tokens come from this
// portion's rows where it holds them and from the ring otherwise.
__device__ __forceinline__ float fh_rec_conv(const FhRecurrent &r, int ch, const float *proj, int64_t ldp, int t, int pos,
                                             const float *ring, int channels) {
    const int nq = r.kv_heads * r.dim;
    const float *w, *b;
    int col, c = ch;
    if (c < nq) w = r.conv_q, b = r.bias_q, col = r.col_q + c;
    else if (c < 2 * nq) c -= nq, w = r.conv_k, b = r.bias_k, col = r.col_k + c;
    else c -= 2 * nq, w = r.conv_v, b = r.bias_v, col = r.col_v + c;
    float acc = 0.f;
    for (int i = 0; i < r.taps; i++) {
        const int tt = t - (r.taps - 1) + i;
        if (pos + tt < 0) continue;
        const float x = tt >= 0 ? proj[(int64_t)tt * ldp + col] : ring[(int64_t)((pos + tt) % r.taps) * channels + ch];
        acc = fmaf(x, w[c * r.taps + i], acc);
    }
    if (b) acc += b[c];
    return fh_silu_f(acc);
}
