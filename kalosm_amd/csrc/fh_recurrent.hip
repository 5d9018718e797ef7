// Prefill of the linear recurrences (fh_recurrent.h): convolutions, rotations and gates of a portion, the recurrence in
// chunks (matrix cores) or token by token, and the gated norm of its output.
#include "fh_recurrent.h"

// ------------------------------------------------------------------------------ inputs of the recurrence
// One workgroup per token.
__global__ __launch_bounds__(256) void k_rec_prep(FhRecurrent r, const float *__restrict__ proj, int64_t ldp, int pos,
                                                  const float *__restrict__ ring, FhRecWork w, int dp) {
    extern __shared__ float qk[]; // [2 * kv_heads * dim]
    const int t = blockIdx.x, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const int nq = r.kv_heads * r.dim, inner = r.heads * r.vdim, channels = 2 * nq + inner;
    for (int ch = tid; ch < channels; ch += 256) {
        const float v = fh_rec_conv(r, ch, proj, ldp, t, pos, ring, channels);
        if (ch < 2 * nq) qk[ch] = v;
        else w.v[(int64_t)t * inner + ch - 2 * nq] = v;
    }
    for (int h = tid; h < r.heads; h += 256) {
        const float *row = proj + (int64_t)t * ldp;
        const float sp = fh_softplus_f(row[r.col_a + h] + r.dt_bias[h]);
        w.la[(int64_t)t * r.heads + h] = -expf(r.a_log[h]) * sp;
        w.beta[(int64_t)t * r.heads + h] = r.delta() ? fh_sigmoid_f(row[r.col_b + h]) : sp;
    }
    __syncthreads();
    for (int h = wave; h < 2 * r.kv_heads; h += 4) {
        const float *x = qk + h * r.dim;
        float f = 1.f;
        if (r.delta()) {
            float ss = 0.f;
            for (int i = lane; i < r.dim; i += 64) ss = fmaf(x[i], x[i], ss);
            f = 1.0f / sqrtf(fh_wave_sum(ss) + 1e-6f);
        }
        if (h < r.kv_heads) f *= r.q_scale;
        float *dst = (h < r.kv_heads ? w.q : w.k) + ((int64_t)t * r.kv_heads + h % r.kv_heads) * dp;
        for (int i = lane; i < dp; i += 64) dst[i] = i < r.dim ? x[i] * f : 0.f;
    }
}

// Retention: rotated queries and keys, values as they are, constant decays.  grid (s, groups of four jobs): one wavefront per
// head of q, of k, of v.
__global__ __launch_bounds__(256) void k_rec_rotate(FhRecurrent r, const float *__restrict__ proj, int64_t ldp, int pos, FhRecWork w, int dp) {
    const int t = blockIdx.x, lane = threadIdx.x & 63, job = (int)blockIdx.y * 4 + (threadIdx.x >> 6), part = job / r.heads, h = job % r.heads;
    const float *row = proj + (int64_t)t * ldp;
    if (part >= 3) return;
    if (part == 2) {
        float *dst = w.v + (int64_t)t * r.heads * r.vdim + h * r.vdim;
        for (int i = lane; i < r.vdim; i += 64) dst[i] = row[r.col_v + h * r.vdim + i];
        if (lane == 0) w.la[(int64_t)t * r.heads + h] = r.log_decay[h], w.beta[(int64_t)t * r.heads + h] = 1.f;
        return;
    }
    const float *ct = r.cos_t + (int64_t)(pos + t) * r.pairs, *st = r.sin_t + (int64_t)(pos + t) * r.pairs;
    const float *x = row + (part ? r.col_k : r.col_q) + h * r.dim, mul = part ? r.k_scale : r.q_scale;
    float *dst = (part ? w.k : w.q) + ((int64_t)t * r.heads + h) * dp;
#pragma unroll 4
    for (int i = lane; i < dp; i += 64)
        dst[i] = i < r.dim ? fh_rotated([&](int j) { return x[j]; }, i, r.pairs, r.halves, ct, st) * mul : 0.f;
}

// Projections of the portion's last `taps` tokens into the ring, after every reader of its old rows.
__global__ void k_rec_tail(FhRecurrent r, const float *__restrict__ proj, int64_t ldp, int s, int pos, float *__restrict__ ring) {
    const int nq = r.kv_heads * r.dim, channels = 2 * nq + r.heads * r.vdim;
    const int ch = blockIdx.x * 256 + threadIdx.x, t = s - 1 - (int)blockIdx.y;
    if (ch >= channels || t < 0) return;
    const int col = ch < nq ? r.col_q + ch : ch < 2 * nq ? r.col_k + ch - nq : r.col_v + ch - 2 * nq;
    ring[(int64_t)((pos + t) % r.taps) * channels + ch] = proj[(int64_t)t * ldp + col];
}

// ------------------------------------------------------------------------------ token by token
// One wavefront per four columns of a head's state; the 16 lanes of a DPP row share a column, RPT consecutive rows each,
// in registers for the whole portion.  The next token's operands are requested before the current one is worked on.
template <int RPT>
__global__ __launch_bounds__(64) void k_rec_scan(FhRecurrent r, FhRecWork w, float *__restrict__ state, int s, int first, int dp) {
    const int h = blockIdx.y, lane = threadIdx.x, rg = lane & 15, col = (int)blockIdx.x * 4 + (lane >> 4);
    const int nq = r.kv_heads * dp, inner = r.heads * r.vdim, kh = h / (r.heads / r.kv_heads), i0 = rg * RPT;
    const bool live = col < r.vdim;
    const int c = live ? col : r.vdim - 1;
    float *sp = state + ((int64_t)h * r.vdim + c) * r.dim;
    float S[RPT], kc[RPT], qc[RPT], kn[RPT], qn[RPT];
#pragma unroll
    for (int i = 0; i < RPT; i++) S[i] = !first && i0 + i < r.dim ? sp[i0 + i] : 0.f;
    const float *kp = w.k + kh * dp + i0, *qp = w.q + kh * dp + i0, *vp = w.v + h * r.vdim + c;
    const float skip = r.d_skip ? r.d_skip[h] : 0.f;
    auto load = [&](int t, float *k, float *q, float &v, float &be, float &la) {
#pragma unroll
        for (int i = 0; i < RPT; i++) {
            k[i] = i0 + i < dp ? kp[(int64_t)t * nq + i] : 0.f;
            q[i] = i0 + i < dp ? qp[(int64_t)t * nq + i] : 0.f;
        }
        v = vp[(int64_t)t * inner];
        be = w.beta[(int64_t)t * r.heads + h];
        la = w.la[(int64_t)t * r.heads + h];
    };
    float v, be, la, vn = 0.f, bn = 0.f, ln = 0.f;
    load(0, kc, qc, v, be, la);
    for (int t = 0; t < s; t++) {
        if (t + 1 < s) load(t + 1, kn, qn, vn, bn, ln);
        const float g = expf(la);
        float dot = 0.f;
#pragma unroll
        for (int i = 0; i < RPT; i++) {
            S[i] *= g;
            dot = fmaf(S[i], kc[i], dot);
        }
        const float u = r.delta() ? be * (v - fh_row16_sum(dot)) : be * v;
        float o = 0.f;
#pragma unroll
        for (int i = 0; i < RPT; i++) {
            S[i] = fmaf(kc[i], u, S[i]);
            o = fmaf(S[i], qc[i], o);
        }
        o = fh_row16_sum(o);
        if (rg == 0 && live) w.o[(int64_t)t * inner + h * r.vdim + col] = o + skip * v;
#pragma unroll
        for (int i = 0; i < RPT; i++) kc[i] = kn[i], qc[i] = qn[i];
        v = vn, be = bn, la = ln;
    }
#pragma unroll
    for (int i = 0; i < RPT; i++)
        if (live && i0 + i < r.dim) sp[i0 + i] = S[i];
}

// The same with one decay per key channel, on rows [t, heads * dim].
template <int RPT>
__global__ __launch_bounds__(64) void k_rec_scan_channel(FhRecurrent r, FhRecRows in, float *__restrict__ out, float *__restrict__ state,
                                                         int s, int first) {
    const int h = blockIdx.y, lane = threadIdx.x, rg = lane & 15, col = (int)blockIdx.x * 4 + (lane >> 4);
    const int inner = r.heads * r.vdim, nq = r.heads * r.dim, i0 = rg * RPT;
    const bool live = col < r.vdim;
    const int c = live ? col : r.vdim - 1;
    float *sp = state + ((int64_t)h * r.vdim + c) * r.dim;
    float S[RPT], u[RPT], w0[RPT];
    struct Ops { float q[RPT], k[RPT], z[RPT], v; } a, b;
#pragma unroll
    for (int i = 0; i < RPT; i++) {
        const bool ok = i0 + i < r.dim;
        S[i] = !first && ok ? sp[i0 + i] : 0.f;
        u[i] = ok ? r.bonus[h * r.dim + i0 + i] : 0.f;
        w0[i] = ok ? r.w0[h * r.dim + i0 + i] : 0.f;
    }
    auto load = [&](int t, Ops &x) {
        const int64_t o = (int64_t)t * nq + h * r.dim + i0;
#pragma unroll
        for (int i = 0; i < RPT; i++) {
            const bool ok = i0 + i < r.dim;
            x.q[i] = ok ? in.q[o + i] : 0.f;
            x.k[i] = ok ? in.k[o + i] : 0.f;
            x.z[i] = ok ? in.z[o + i] : 0.f;
        }
        x.v = in.v[(int64_t)t * inner + h * r.vdim + c];
    };
    load(0, a);
    for (int t = 0; t < s; t++) {
        load(t + 1 < s ? t + 1 : t, b);
        float o = 0.f;
#pragma unroll
        for (int i = 0; i < RPT; i++) {
            const float kv = a.k[i] * a.v;
            o = fmaf(fmaf(u[i], kv, S[i]), a.q[i], o);
            S[i] = fmaf(S[i], expf(fh_rec_la(a.z[i] + w0[i])), kv);
        }
        o = fh_row16_sum(o);
        if (rg == 0 && live) out[(int64_t)t * inner + h * r.vdim + col] = o;
        a = b;
    }
#pragma unroll
    for (int i = 0; i < RPT; i++)
        if (live && i0 + i < r.dim) sp[i0 + i] = S[i];
}

// ------------------------------------------------------------------------------ gated norm
template <typename T>
__global__ __launch_bounds__(256) void k_rec_out(FhRecurrent r, const float *__restrict__ o, const float *__restrict__ gates,
                                                 int64_t ldg, T *__restrict__ y, int ldy, int kp) {
    extern __shared__ float xs[]; // [inner]
    const int t = blockIdx.x, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, inner = r.heads * r.vdim;
    const float *gate = gates + (int64_t)t * ldg, *orow = o + (int64_t)t * inner;
    for (int i = tid; i < inner; i += 256) {
        float v = orow[i];
        if (r.gate_first) v *= fh_silu_f(gate[i]);
        xs[i] = v;
    }
    __syncthreads();
    const int gl = inner / r.norm_groups;
    T *yr = y + (int64_t)t * ldy;
    for (int g = wave; g < r.norm_groups; g += 4) {
        float ss = 0.f;
        for (int i = lane; i < gl; i += 64) ss = fmaf(xs[g * gl + i], xs[g * gl + i], ss);
        const float inv = 1.0f / sqrtf(fh_wave_sum(ss) / (float)gl + r.eps);
        for (int i = lane; i < gl; i += 64) {
            const int c = g * gl + i;
            float v = xs[c] * inv;
            if (r.norm) v *= r.norm[r.norm_len == inner ? c : c % r.norm_len];
            if (!r.gate_first) v *= fh_silu_f(gate[c]);
            yr[c] = fh_to<T>(v * r.out_scale);
        }
    }
    for (int i = inner + tid; i < kp; i += 256) yr[i] = fh_to<T>(0.f);
}

// ------------------------------------------------------------------------------ in chunks of 64 tokens
// With c_t the running sum of la inside a chunk and S the state before it:
//   O = e^c Q S + M U,   M_ts = e^(c_t - c_s) q_t . k_s  (s <= t),   S <- e^c_63 S + sum_s e^(c_63 - c_s) k_s u_s^T
//   state space, retention: u_t = beta_t v_t
//   delta rule:  (1 + L) U = beta V - beta e^c K S,   L_ts = beta_t e^(c_t - c_s) k_t . k_s  (s < t)
// The first launch works on all chunks at once: M, K^T, and for the delta rule U0 = (1 + L)^-1 beta V and
// W = (1 + L)^-1 beta e^c K by forward substitution, one column of [W | U0] per thread with the 64 rows in registers.
// Channel decay, with C_t the running sum of the la of a channel:
//   O = (e^(C_(t-1)) q) S + M V,   M_ts = sum_c q_tc k_sc e^(C_(t-1)c - C_sc) (s < t),  M_tt = sum_c q_tc bonus_c k_tc
//   S <- e^C_63 S + sum_s (e^(C_63 - C_s) k_s) v_s^T
// No exponent may be positive, or fast decays would overflow: blocks of M below the diagonal ones split theirs at the start
// of the row block, the diagonal blocks are summed pair by pair.
// The second walks the chunks with 16 columns of a head's state per workgroup: U = U0 - W S.  All products are
// v_mfma_f32_16x16x4_f32; a lane takes four neighbouring k of an operand row at a time, on both sides alike.
struct RecChunks { // scratch of one portion
    float *m, *w, *u0; // per (chunk, head): [64][64], [64][dp], [64][vp]
    float *kt;         // per (chunk, key head): [dp][64]
    float *q, *f;      // channel decay, per (chunk, head): [64][dp] queries with the decay from the chunk's start, [dp] that of the chunk
    int dp, vp, n;     // vp: vdim rounded up to 16, n: chunks
};
static RecChunks rec_chunks(const FhRecurrent &r, int s, float *p) {
    RecChunks c{};
    c.dp = fh_rec_dp(r), c.vp = (r.vdim + 15) / 16 * 16, c.n = (s + 63) / 64;
    const size_t hc = (size_t)c.n * r.heads;
    c.m = p, p += hc * 4096;
    c.kt = p, p += (size_t)c.n * r.kv_heads * c.dp * 64;
    if (r.delta()) c.w = p, p += hc * 64 * c.dp, c.u0 = p;
    if (r.kind == FH_REC_CHANNEL) c.q = p, p += hc * 64 * c.dp, c.f = p;
    return c;
}
size_t fh_rec_chunk_floats(const FhRecurrent &r, int s) {
    const RecChunks c = rec_chunks(r, s, nullptr);
    return (size_t)c.n * ((size_t)r.heads * (4096 + (r.delta() ? 64 * (c.dp + c.vp) : r.kind == FH_REC_CHANNEL ? 65 * c.dp : 0)) + (size_t)r.kv_heads * c.dp * 64);
}

__device__ __forceinline__ fh_f4 mma4(const float4 &a, const float4 &b, fh_f4 c) { // 16 of k
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b.x, c, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b.y, c, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b.z, c, 0, 0, 0);
    return __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b.w, c, 0, 0, 0);
}
// Running sum of la over the 64 tokens of a chunk (one wavefront; tokens past the end change nothing).
__device__ __forceinline__ float rec_decay_sum(const FhRecWork &w, int t, int s, int heads, int h) {
    float v = t < s ? w.la[(int64_t)t * heads + h] : 0.f;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
        const float u = __shfl_up(v, o, 64);
        if ((int)(threadIdx.x & 63) >= o) v += u;
    }
    return v;
}

template <int DP, bool DELTA>
__global__ __launch_bounds__(256) void k_rec_chunk_prep(FhRecurrent r, FhRecWork w, RecChunks c, int s) {
    constexpr int LD = DP + 4, LL = 68;
    extern __shared__ __attribute__((aligned(16))) float lds[];
    float *sk = lds, *sq = sk + 64 * LD, *cs = sq + 64 * (LD > LL ? LD : LL), *be = cs + 64; // L takes the place of Q
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, li = lane & 15, g = lane >> 4;
    const int ch = blockIdx.x, h = blockIdx.y, rep = r.heads / r.kv_heads, kh = h / rep, t0 = ch * 64;
    for (int i = tid; i < 64 * DP / 4; i += 256) {
        const int t = i / (DP / 4), x = i % (DP / 4) * 4;
        const int64_t o = ((int64_t)(t0 + t) * r.kv_heads + kh) * DP + x;
        const float4 z = make_float4(0.f, 0.f, 0.f, 0.f);
        *(float4 *)(sk + t * LD + x) = t0 + t < s ? *(const float4 *)(w.k + o) : z;
        *(float4 *)(sq + t * LD + x) = t0 + t < s ? *(const float4 *)(w.q + o) : z;
    }
    if (wave == 0) {
        cs[lane] = rec_decay_sum(w, t0 + lane, s, r.heads, h);
        be[lane] = t0 + lane < s ? w.beta[(int64_t)(t0 + lane) * r.heads + h] : 0.f;
    }
    __syncthreads();
    const int64_t hc = (int64_t)ch * r.heads + h;
    float *mo = c.m + hc * 4096;
    fh_f4 kk[4];
#pragma unroll
    for (int b = 0; b < 4; b++) { // wavefront: rows 16 wave .. + 15 against the 16 tokens of block b <= wave
        if (b > wave) break;
        fh_f4 qk = fh_f4{0.f, 0.f, 0.f, 0.f};
        kk[b] = qk;
#pragma unroll
        for (int x = 0; x < DP / 16; x++) {
            const float4 kb = *(const float4 *)(sk + (16 * b + li) * LD + 16 * x + 4 * g);
            qk = mma4(*(const float4 *)(sq + (16 * wave + li) * LD + 16 * x + 4 * g), kb, qk);
            if (DELTA) kk[b] = mma4(*(const float4 *)(sk + (16 * wave + li) * LD + 16 * x + 4 * g), kb, kk[b]);
        }
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int t = 16 * wave + 4 * g + e, u = 16 * b + li;
            mo[t * 64 + u] = u <= t ? expf(cs[t] - cs[u]) * qk[e] : 0.f;
        }
    }
    if (h % rep == 0) {
        float *kt = c.kt + ((int64_t)ch * r.kv_heads + kh) * DP * 64;
        for (int i = tid; i < DP * 64; i += 256) kt[i] = sk[(i & 63) * LD + (i >> 6)];
    }
    if (!DELTA) return;
    __syncthreads(); // Q has been read
    float *sl = sq;
#pragma unroll
    for (int b = 0; b < 4; b++) {
        if (b > wave) break;
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int t = 16 * wave + 4 * g + e, u = 16 * b + li;
            sl[t * LL + u] = u < t ? be[t] * expf(cs[t] - cs[u]) * kk[b][e] : 0.f;
        }
    }
    __syncthreads();
    for (int j = tid; j < DP + c.vp; j += 256) {
        float x[64];
        if (j < DP) {
#pragma unroll
            for (int t = 0; t < 64; t++) x[t] = be[t] * expf(cs[t]) * sk[t * LD + j];
        } else {
            const int col = j - DP;
#pragma unroll
            for (int t = 0; t < 64; t++)
                x[t] = t0 + t < s && col < r.vdim ? be[t] * w.v[((int64_t)(t0 + t) * r.heads + h) * r.vdim + col] : 0.f;
        }
#pragma unroll
        for (int t = 1; t < 64; t++) {
            float a = x[t];
#pragma unroll
            for (int u = 0; u < (t + 3) / 4; u++) {
                const float4 l = *(const float4 *)(sl + t * LL + 4 * u); // zeros from u = t on inside the diagonal block
                a = fmaf(-l.x, x[4 * u], a);
                if (4 * u + 1 < t) a = fmaf(-l.y, x[4 * u + 1], a);
                if (4 * u + 2 < t) a = fmaf(-l.z, x[4 * u + 2], a);
                if (4 * u + 3 < t) a = fmaf(-l.w, x[4 * u + 3], a);
            }
            x[t] = a;
        }
        float *dst = j < DP ? c.w + hc * 64 * DP + j : c.u0 + hc * 64 * c.vp + j - DP;
        const int st = j < DP ? DP : c.vp;
#pragma unroll
        for (int t = 0; t < 64; t++) dst[t * st] = x[t];
    }
}

// Channel decay: one workgroup per (chunk, head).  Sums of la start anew in every block of 16 tokens, so that a fast decay
// ahead of a block takes no digits from the sums inside it; longer ones are put together from those.  They are base-2
// logarithms: no exponent is positive, so that v_exp_f32 does as it is (results below 2^-126 count as zero).
__device__ __forceinline__ float rec_exp2(float x) { return __builtin_amdgcn_exp2f(x); }
template <int DP>
__global__ __launch_bounds__(256) void k_rec_channel_prep(FhRecurrent r, FhRecRows in, RecChunks c, int s) {
    constexpr int LD = DP + 4;
    extern __shared__ __attribute__((aligned(16))) float lds[];
    float *sk = lds, *sq = sk + 64 * LD, *sc = sq + 64 * LD, *ub = sc + 68 * LD; // sc row 17 b + i: la of the first i tokens of block b
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, li = lane & 15, g = lane >> 4;
    const int ch = blockIdx.x, h = blockIdx.y, t0 = ch * 64, nq = r.heads * r.dim;
    const int64_t hc = (int64_t)ch * r.heads + h;
    constexpr int B = 8; // requests of a thread and array on their way; places outside read a valid address
    for (int i0 = tid; i0 < 64 * DP; i0 += 256 * B) {
        float k[B], q[B], z[B];
#pragma unroll
        for (int j = 0; j < B; j++) {
            const int i = i0 + 256 * j, t = t0 + i / DP, x = i % DP;
            const int64_t o = (int64_t)(t < s ? t : s - 1) * nq + h * r.dim + (x < r.dim ? x : r.dim - 1);
            k[j] = in.k[o], q[j] = in.q[o], z[j] = in.z[o];
        }
#pragma unroll
        for (int j = 0; j < B; j++) {
            const int i = i0 + 256 * j, t = i / DP, x = i % DP;
            const bool ok = t0 + t < s && x < r.dim;
            sk[t * LD + x] = ok ? k[j] : 0.f;
            sq[t * LD + x] = ok ? q[j] : 0.f;
            // nothing is forgotten past the end
            sc[(t / 16 * 17 + t % 16 + 1) * LD + x] = ok ? fh_rec_la(z[j] + r.w0[h * r.dim + x]) * 1.4426950408889634f : 0.f;
        }
    }
    for (int x = tid; x < DP; x += 256) ub[x] = x < r.dim ? r.bonus[h * r.dim + x] : 0.f;
    __syncthreads();
    for (int i = tid; i < 4 * DP; i += 256) {
        float *p = sc + i / DP * 17 * LD + i % DP, v = 0.f;
        p[0] = 0.f;
#pragma unroll
        for (int t = 1; t <= 16; t++) p[t * LD] = v += p[t * LD];
    }
    __syncthreads();
    // la of block b behind its first i tokens, of the whole blocks from b0 to b1 - 1
    auto rest = [&](int b, int i, int x) { return sc[(17 * b + 16) * LD + x] - sc[(17 * b + i) * LD + x]; };
    auto blocks = [&](int b0, int b1, int x) {
        float v = 0.f;
        for (int b = b0; b < b1; b++) v += sc[(17 * b + 16) * LD + x];
        return v;
    };
    float *mo = c.m + hc * 4096;
    fh_f4 off[3];
#pragma unroll
    for (int b = 0; b < 3; b++) off[b] = fh_f4{0.f, 0.f, 0.f, 0.f};
    if (wave > 0)
#pragma unroll
        for (int x = 0; x < DP / 16; x++) {
            const int o = 16 * x + 4 * g, t = 16 * wave + li;
            const float4 cq = *(const float4 *)(sc + (17 * wave + li) * LD + o), q = *(const float4 *)(sq + t * LD + o);
            const float4 qa = make_float4(q.x * rec_exp2(cq.x), q.y * rec_exp2(cq.y), q.z * rec_exp2(cq.z), q.w * rec_exp2(cq.w));
#pragma unroll
            for (int b = 0; b < 3; b++) {
                if (b >= wave) break;
                const float4 k = *(const float4 *)(sk + (16 * b + li) * LD + o);
                float f[4];
#pragma unroll
                for (int e = 0; e < 4; e++) f[e] = rec_exp2(rest(b, li + 1, o + e) + blocks(b + 1, wave, o + e));
                off[b] = mma4(qa, make_float4(k.x * f[0], k.y * f[1], k.z * f[2], k.w * f[3]), off[b]);
            }
        }
#pragma unroll
    for (int b = 0; b < 3; b++) {
        if (b >= wave) break;
#pragma unroll
        for (int e = 0; e < 4; e++) mo[(16 * wave + 4 * g + e) * 64 + 16 * b + li] = off[b][e];
    }
#pragma unroll
    for (int e = 0; e < 4; e++) {
        const int t = 16 * wave + 4 * g + e, u = 16 * wave + li;
        float a = 0.f;
        if (u <= t)
            for (int x = 0; x < DP; x += 4) {
                const float4 q = *(const float4 *)(sq + t * LD + x), k = *(const float4 *)(sk + u * LD + x);
                float4 f;
                if (u == t) f = *(const float4 *)(ub + x);
                else {
                    const float4 ct = *(const float4 *)(sc + (17 * wave + 4 * g + e) * LD + x), cu = *(const float4 *)(sc + (17 * wave + li + 1) * LD + x);
                    f = make_float4(rec_exp2(ct.x - cu.x), rec_exp2(ct.y - cu.y), rec_exp2(ct.z - cu.z), rec_exp2(ct.w - cu.w));
                }
                a = fmaf(q.x * k.x, f.x, fmaf(q.y * k.y, f.y, fmaf(q.z * k.z, f.z, fmaf(q.w * k.w, f.w, a))));
            }
        mo[t * 64 + u] = a;
    }
    for (int i = tid; i < 64 * DP; i += 256) {
        const int t = i / DP, x = i % DP;
        c.q[(hc * 64 + t) * DP + x] = sq[t * LD + x] * rec_exp2(blocks(0, t / 16, x) + sc[(t / 16 * 17 + t % 16) * LD + x]);
    }
    for (int i = tid; i < DP * 64; i += 256) {
        const int t = i & 63, x = i >> 6;
        c.kt[hc * DP * 64 + i] = sk[t * LD + x] * rec_exp2(rest(t / 16, t % 16 + 1, x) + blocks(t / 16 + 1, 4, x));
    }
    for (int x = tid; x < DP; x += 256) c.f[hc * DP + x] = rec_exp2(blocks(0, 4, x));
}

// grid (blocks of 16 value columns, heads), four wavefronts.  Wavefront w works out rows 16 w .. + 15 of U and O and rows
// DP / 4 w .. of the state; U and the state pass between the wavefronts through the LDS, one column per row.
template <int DP, int KIND>
__global__ __launch_bounds__(256, 1) void k_rec_chunk_scan(FhRecurrent r, FhRecWork w, RecChunks c, float *__restrict__ state, int s,
                                                           int first) {
    constexpr bool DELTA = KIND == FH_REC_DELTA, CHANNEL = KIND == FH_REC_CHANNEL;
    constexpr int ST = DP / 64 > 0 ? DP / 64 : 1, SL = DP + 4, UL = 68; // state tiles of a wavefront
    constexpr int SW = DP / 16 / ST;                                    // wavefronts with state rows
    __shared__ __attribute__((aligned(16))) float ss[16 * SL], su[16 * UL], sd[16 * UL], cs[2][64];
    const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, li = lane & 15, g = lane >> 4;
    // The column blocks of a head read the same operands: they go to one of the eight dies, whose L2 then serves all but one
    // (workgroups are dealt to the dies in turn).
    const int ncb = c.vp / 16, lin = blockIdx.x, full = r.heads / 8 * 8 * ncb;
    const int h = lin < full ? lin % 8 + lin / (8 * ncb) * 8 : lin / ncb, cb = lin < full ? lin / 8 % ncb : lin % ncb;
    const int kh = h / (r.heads / r.kv_heads), col = cb * 16 + li;
    const bool live = col < r.vdim, owner = wave < SW;
    float *sp = state + ((int64_t)h * r.vdim + (live ? col : r.vdim - 1)) * r.dim;
    fh_f4 S[ST];
#pragma unroll
    for (int i = 0; i < ST; i++)
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int row = (wave * ST + i) * 16 + 4 * g + e;
            S[i][e] = !first && live && owner && row < r.dim ? sp[row] : 0.f;
        }
    const float skip = r.d_skip ? r.d_skip[h] : 0.f;
    struct Ops { // a lane's operands of one chunk
        float4 w[DELTA ? DP / 16 : 1], q[DP / 16], m[4], kt[ST][4];
        float u[4], v[4], la;
        float4 f[CHANNEL ? ST : 1];
    } o0, o1;
    // No branches around the requests: the number in flight is then known at compile time, so that waiting for one chunk's
    // operands does not wait for the next one's.  Places outside the portion read a valid address instead.
    auto load = [&](Ops &o, int ch) {
        const int64_t hc = (int64_t)ch * r.heads + h;
        const int t = ch * 64 + 16 * wave + li, tq = t < s ? t : s - 1; // rows past the end are multiplied by zeros of M and decays
        if (DELTA) {
            const float *wp = c.w + (hc * 64 + 16 * wave + li) * DP + 4 * g;
#pragma unroll
            for (int x = 0; x < DP / 16; x++) o.w[x] = *(const float4 *)(wp + 16 * x);
        }
        const float *qp = (CHANNEL ? c.q + (hc * 64 + 16 * wave + li) * DP : w.q + ((int64_t)tq * r.kv_heads + kh) * DP) + 4 * g;
#pragma unroll
        for (int x = 0; x < DP / 16; x++) o.q[x] = *(const float4 *)(qp + 16 * x);
        const float *mp = c.m + hc * 4096 + (16 * wave + li) * 64 + 4 * g;
#pragma unroll
        for (int b = 0; b < 4; b++) o.m[b] = *(const float4 *)(mp + 16 * b); // blocks behind the diagonal are never used
        const float *kp = c.kt + (((int64_t)ch * r.kv_heads + kh) * DP + (owner ? wave : 0) * ST * 16 + li) * 64 + 4 * g;
#pragma unroll
        for (int i = 0; i < ST; i++)
#pragma unroll
            for (int b = 0; b < 4; b++) o.kt[i][b] = *(const float4 *)(kp + i * 1024 + 16 * b);
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int row = 16 * wave + 4 * g + e, tt = ch * 64 + row < s ? ch * 64 + row : s - 1;
            if (CHANNEL) o.v[e] = w.v[((int64_t)tt * r.heads + h) * r.vdim + (live ? col : r.vdim - 1)];
            else if (DELTA) o.u[e] = c.u0[(hc * 64 + row) * c.vp + col];
            else {
                o.v[e] = w.v[((int64_t)tt * r.heads + h) * r.vdim + (live ? col : r.vdim - 1)];
                o.u[e] = w.beta[(int64_t)tt * r.heads + h];
            }
        }
        if (CHANNEL)
#pragma unroll
            for (int i = 0; i < ST; i++) o.f[i] = *(const float4 *)(c.f + hc * DP + (owner ? wave : 0) * ST * 16 + i * 16 + 4 * g);
        else o.la = w.la[(int64_t)(ch * 64 + lane < s ? ch * 64 + lane : s - 1) * r.heads + h];
    };
    auto step = [&](const Ops &o, int ch) {
        float *c_ = cs[ch & 1];
        if (!CHANNEL && wave == 0) {
            float v = ch * 64 + lane < s ? o.la : 0.f;
#pragma unroll
            for (int d = 1; d < 64; d <<= 1) {
                const float u = __shfl_up(v, d, 64);
                if (lane >= d) v += u;
            }
            c_[lane] = v;
        }
        if (owner)
#pragma unroll
            for (int i = 0; i < ST; i++) *(fh_f4 *)(ss + li * SL + (wave * ST + i) * 16 + 4 * g) = S[i];
        __syncthreads(); // state and decays are there; U of the chunk before has been read
        fh_f4 ws = fh_f4{0.f, 0.f, 0.f, 0.f}, qs = ws;
#pragma unroll
        for (int x = 0; x < DP / 16; x++) {
            const float4 b = *(const float4 *)(ss + li * SL + 16 * x + 4 * g);
            if (DELTA) ws = mma4(o.w[x], b, ws);
            qs = mma4(o.q[x], b, qs);
        }
        const float end = CHANNEL ? 0.f : c_[63];
        fh_f4 u, ud, out;
#pragma unroll
        for (int e = 0; e < 4; e++) {
            if (CHANNEL) { // decays are in the operands
                ud[e] = u[e] = ch * 64 + 16 * wave + 4 * g + e < s ? o.v[e] : 0.f;
                out[e] = qs[e];
                continue;
            }
            const float ct = c_[16 * wave + 4 * g + e];
            u[e] = DELTA ? o.u[e] - ws[e] : ch * 64 + 16 * wave + 4 * g + e < s ? o.u[e] * o.v[e] : 0.f;
            ud[e] = expf(end - ct) * u[e];
            out[e] = expf(ct) * qs[e];
        }
        *(fh_f4 *)(su + li * UL + 16 * wave + 4 * g) = u;
        if (!CHANNEL) *(fh_f4 *)(sd + li * UL + 16 * wave + 4 * g) = ud;
        __syncthreads();
#pragma unroll
        for (int b = 0; b < 4; b++)
            if (b <= wave) out = mma4(o.m[b], *(const float4 *)(su + li * UL + 16 * b + 4 * g), out);
        const float f = CHANNEL ? 1.f : expf(end), *su_ = CHANNEL ? su : sd;
        if (owner)
#pragma unroll
            for (int i = 0; i < ST; i++) {
#pragma unroll
                for (int e = 0; e < 4; e++) S[i][e] *= !CHANNEL ? f : e == 0 ? o.f[i].x : e == 1 ? o.f[i].y : e == 2 ? o.f[i].z : o.f[i].w;
#pragma unroll
                for (int b = 0; b < 4; b++) S[i] = mma4(o.kt[i][b], *(const float4 *)(su_ + li * UL + 16 * b + 4 * g), S[i]);
            }
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int tt = ch * 64 + 16 * wave + 4 * g + e;
            if (tt < s && live) w.o[((int64_t)tt * r.heads + h) * r.vdim + col] = DELTA || CHANNEL ? out[e] : out[e] + skip * o.v[e];
        }
    };
    load(o0, 0);
    for (int ch = 0; ch < c.n; ch += 2) { // the next chunk's operands are requested before the current one is worked on
        load(o1, ch + 1 < c.n ? ch + 1 : ch);
        step(o0, ch);
        if (ch + 1 >= c.n) break;
        load(o0, ch + 2 < c.n ? ch + 2 : ch);
        step(o1, ch + 1);
    }
#pragma unroll
    for (int i = 0; i < ST; i++)
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int row = (wave * ST + i) * 16 + 4 * g + e;
            if (live && owner && row < r.dim) sp[row] = S[i][e];
        }
}

template <int DP, bool DELTA>
static fh_status rec_chunked(fh_device *dev, const FhRecurrent &r, const FhRecWork &w, float *state, int s, bool first) {
    const RecChunks c = rec_chunks(r, s, w.chunk);
    const size_t lds = (size_t)(64 * (DP + 4) + 64 * (DP + 4 > 68 ? DP + 4 : 68) + 128) * 4;
    auto prep = k_rec_chunk_prep<DP, DELTA>;
    if (lds > 48 * 1024) FH_TRY(fh_kernel_lds(dev, (const void *)prep, lds));
    prep<<<dim3((unsigned)c.n, (unsigned)r.heads), 256, lds, dev->stream>>>(r, w, c, s);
    k_rec_chunk_scan<DP, DELTA ? FH_REC_DELTA : FH_REC_SPACE><<<dim3((unsigned)(c.vp / 16 * r.heads)), 256, 0, dev->stream>>>(r, w, c, state, s, first);
    FH_HIP(hipGetLastError());
    return FH_OK;
}

template <int DP>
static fh_status rec_channel_chunked(fh_device *dev, const FhRecurrent &r, const FhRecRows &in, const FhRecWork &w, float *state, int s, bool first) {
    const RecChunks c = rec_chunks(r, s, w.chunk);
    const size_t lds = (size_t)(196 * (DP + 4) + DP) * 4;
    if (lds > 48 * 1024) FH_TRY(fh_kernel_lds(dev, (const void *)k_rec_channel_prep<DP>, lds));
    k_rec_channel_prep<DP><<<dim3((unsigned)c.n, (unsigned)r.heads), 256, lds, dev->stream>>>(r, in, c, s);
    k_rec_chunk_scan<DP, FH_REC_CHANNEL><<<dim3((unsigned)(c.vp / 16 * r.heads)), 256, 0, dev->stream>>>(r, w, c, state, s, first);
    FH_HIP(hipGetLastError());
    return FH_OK;
}

static fh_status rec_out(fh_device *dev, int dtype, const FhRecurrent &r, const float *o, const float *gates, int64_t ldg, int s, void *y,
                         int ldy, int kp) {
    const size_t lds = (size_t)fh_rec_inner(r) * 4;
    FH_REQUIRE(lds <= 150 * 1024, "recurrent layer of %d channels is too wide", fh_rec_inner(r));
    const dim3 grid((unsigned)s);
    if (dtype == FH_F32) {
        if (lds > 48 * 1024) FH_TRY(fh_kernel_lds(dev, (const void *)k_rec_out<float>, lds));
        k_rec_out<float><<<grid, 256, lds, dev->stream>>>(r, o, gates, ldg, (float *)y, ldy, kp);
    } else {
        if (lds > 48 * 1024) FH_TRY(fh_kernel_lds(dev, (const void *)k_rec_out<uint16_t>, lds));
        k_rec_out<uint16_t><<<grid, 256, lds, dev->stream>>>(r, o, gates, ldg, (uint16_t *)y, ldy, kp);
    }
    FH_HIP(hipGetLastError());
    return FH_OK;
}

fh_status fh_recurrent_channel(fh_device *dev, int dtype, const FhRecurrent &r, const FhRecState &st, const FhRecRows &in, int s, int pos,
                               const FhRecWork &work, void *y, int ldy, int kp) {
    FhRecWork w = work;
    w.v = const_cast<float *>(in.v); // only read
    const int rpt = (r.dim + 15) / 16;
    const int64_t kernel = dev->opt_recurrent_kernel;
    const bool first = pos == 0;
    if (r.dim <= 128 && (kernel == 2 || (kernel == 0 && s >= 24))) { // a wider head's three arrays do not fit the LDS
        switch (fh_rec_dp(r)) {
        case 32: FH_TRY(rec_channel_chunked<32>(dev, r, in, w, st.s, s, first)); break;
        case 64: FH_TRY(rec_channel_chunked<64>(dev, r, in, w, st.s, s, first)); break;
        default: FH_TRY(rec_channel_chunked<128>(dev, r, in, w, st.s, s, first)); break;
        }
    } else {
        const dim3 g((unsigned)((r.vdim + 3) / 4), (unsigned)r.heads);
        FH_REQUIRE(rpt <= 16, "recurrent state of %d rows (at most 256)", r.dim);
        if (rpt <= 2) k_rec_scan_channel<2><<<g, 64, 0, dev->stream>>>(r, in, w.o, st.s, s, first);
        else if (rpt <= 4) k_rec_scan_channel<4><<<g, 64, 0, dev->stream>>>(r, in, w.o, st.s, s, first);
        else if (rpt <= 8) k_rec_scan_channel<8><<<g, 64, 0, dev->stream>>>(r, in, w.o, st.s, s, first);
        else k_rec_scan_channel<16><<<g, 64, 0, dev->stream>>>(r, in, w.o, st.s, s, first);
    }
    return rec_out(dev, dtype, r, w.o, in.g, r.heads * r.vdim, s, y, ldy, kp);
}

fh_status fh_recurrent_prefill(fh_device *dev, int dtype, const FhRecurrent &r, const FhRecState &st, const float *proj,
                               int64_t ldp, int s, int pos, const FhRecWork &w, void *y, int kp) {
    hipStream_t str = dev->stream;
    const int dp = fh_rec_dp(r);
    if (r.kind == FH_REC_RETENTION) k_rec_rotate<<<dim3((unsigned)s, (unsigned)((3 * r.heads + 3) / 4)), 256, 0, str>>>(r, proj, ldp, pos, w, dp);
    else {
        const int nq = r.kv_heads * r.dim, channels = fh_rec_channels(r);
        const size_t lds = (size_t)2 * nq * 4;
        FH_REQUIRE(lds <= 150 * 1024, "recurrent layer of %d channels is too wide", channels);
        if (lds > 48 * 1024) FH_TRY(fh_kernel_lds(dev, (const void *)k_rec_prep, lds));
        k_rec_prep<<<dim3((unsigned)s), 256, lds, str>>>(r, proj, ldp, pos, st.conv, w, dp);
        const int ty = s < r.taps ? s : r.taps;
        k_rec_tail<<<dim3((unsigned)((channels + 255) / 256), (unsigned)ty), 256, 0, str>>>(r, proj, ldp, s, pos, st.conv);
    }
    const dim3 sg((unsigned)((r.vdim + 3) / 4), (unsigned)r.heads);
    const int rpt = (r.dim + 15) / 16;
    const int64_t kernel = dev->opt_recurrent_kernel;
    if (kernel == 2 || (kernel == 0 && s >= 24)) {
        const bool f = pos == 0;
        switch (dp) {
        case 32: FH_TRY(r.delta() ? (rec_chunked<32, true>(dev, r, w, st.s, s, f)) : (rec_chunked<32, false>(dev, r, w, st.s, s, f))); break;
        case 64: FH_TRY(r.delta() ? (rec_chunked<64, true>(dev, r, w, st.s, s, f)) : (rec_chunked<64, false>(dev, r, w, st.s, s, f))); break;
        case 128: FH_TRY(r.delta() ? (rec_chunked<128, true>(dev, r, w, st.s, s, f)) : (rec_chunked<128, false>(dev, r, w, st.s, s, f))); break;
        default: FH_TRY(r.delta() ? (rec_chunked<256, true>(dev, r, w, st.s, s, f)) : (rec_chunked<256, false>(dev, r, w, st.s, s, f))); break;
        }
    } else if (rpt <= 2) k_rec_scan<2><<<sg, 64, 0, str>>>(r, w, st.s, s, pos == 0, dp);
    else if (rpt <= 4) k_rec_scan<4><<<sg, 64, 0, str>>>(r, w, st.s, s, pos == 0, dp);
    else if (rpt <= 8) k_rec_scan<8><<<sg, 64, 0, str>>>(r, w, st.s, s, pos == 0, dp);
    else if (rpt <= 16) k_rec_scan<16><<<sg, 64, 0, str>>>(r, w, st.s, s, pos == 0, dp);
    else FH_FAIL(FH_ERR_UNSUPPORTED, "recurrent state of %d rows (at most 256)", r.dim);
    FH_HIP(hipGetLastError());
    return rec_out(dev, dtype, r, w.o, proj + r.col_g, ldp, s, y, kp, kp);
}
