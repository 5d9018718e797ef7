// Prefill of the gated linear recurrences (fh_recurrent.h): convolutions and gates of a portion, the recurrence token by
// token, and the gated norm of its output.
#include "fh_recurrent.h"

// ------------------------------------------------------------------------------ inputs of the recurrence
// One workgroup per token.
__global__ __launch_bounds__(256) void k_rec_prep(FhRecurrent r, const float *__restrict__ proj, int64_t ldp, int pos,
                                                  const float *__restrict__ ring, FhRecWork w) {
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
        w.beta[(int64_t)t * r.heads + h] = r.delta ? fh_sigmoid_f(row[r.col_b + h]) : sp;
    }
    __syncthreads();
    for (int h = wave; h < 2 * r.kv_heads; h += 4) {
        const float *x = qk + h * r.dim;
        float f = 1.f;
        if (r.delta) {
            float ss = 0.f;
            for (int i = lane; i < r.dim; i += 64) ss = fmaf(x[i], x[i], ss);
            f = 1.0f / sqrtf(fh_wave_sum(ss) + 1e-6f);
        }
        if (h < r.kv_heads) f *= r.q_scale;
        float *dst = (h < r.kv_heads ? w.q : w.k) + (int64_t)t * nq + (h % r.kv_heads) * r.dim;
        for (int i = lane; i < r.dim; i += 64) dst[i] = x[i] * f;
    }
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
__global__ __launch_bounds__(64) void k_rec_scan(FhRecurrent r, FhRecWork w, float *__restrict__ state, int s, int first) {
    const int h = blockIdx.y, lane = threadIdx.x, rg = lane & 15, col = (int)blockIdx.x * 4 + (lane >> 4);
    const int nq = r.kv_heads * r.dim, inner = r.heads * r.vdim, kh = h / (r.heads / r.kv_heads), i0 = rg * RPT;
    const bool live = col < r.vdim;
    const int c = live ? col : r.vdim - 1;
    float *sp = state + ((int64_t)h * r.vdim + c) * r.dim;
    float S[RPT], kc[RPT], qc[RPT], kn[RPT], qn[RPT];
#pragma unroll
    for (int i = 0; i < RPT; i++) S[i] = !first && i0 + i < r.dim ? sp[i0 + i] : 0.f;
    const float *kp = w.k + kh * r.dim + i0, *qp = w.q + kh * r.dim + i0, *vp = w.v + h * r.vdim + c;
    const float skip = r.d_skip ? r.d_skip[h] : 0.f;
    auto load = [&](int t, float *k, float *q, float &v, float &be, float &la) {
#pragma unroll
        for (int i = 0; i < RPT; i++) {
            k[i] = i0 + i < r.dim ? kp[(int64_t)t * nq + i] : 0.f;
            q[i] = i0 + i < r.dim ? qp[(int64_t)t * nq + i] : 0.f;
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
        const float u = r.delta ? be * (v - fh_row16_sum(dot)) : be * v;
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

// ------------------------------------------------------------------------------ gated norm
template <typename T>
__global__ __launch_bounds__(256) void k_rec_out(FhRecurrent r, const float *__restrict__ o, const float *__restrict__ proj,
                                                 int64_t ldp, T *__restrict__ y, int kp) {
    extern __shared__ float xs[]; // [inner]
    const int t = blockIdx.x, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, inner = r.heads * r.vdim;
    const float *gate = proj + (int64_t)t * ldp + r.col_g, *orow = o + (int64_t)t * inner;
    for (int i = tid; i < inner; i += 256) {
        float v = orow[i];
        if (r.gate_first) v *= fh_silu_f(gate[i]);
        xs[i] = v;
    }
    __syncthreads();
    const int gl = inner / r.norm_groups;
    T *yr = y + (int64_t)t * kp;
    for (int g = wave; g < r.norm_groups; g += 4) {
        float ss = 0.f;
        for (int i = lane; i < gl; i += 64) ss = fmaf(xs[g * gl + i], xs[g * gl + i], ss);
        const float inv = 1.0f / sqrtf(fh_wave_sum(ss) / (float)gl + r.eps);
        for (int i = lane; i < gl; i += 64) {
            const int c = g * gl + i;
            float v = xs[c] * inv * r.norm[r.norm_len == inner ? c : c % r.norm_len];
            if (!r.gate_first) v *= fh_silu_f(gate[c]);
            yr[c] = fh_to<T>(v);
        }
    }
    for (int i = inner + tid; i < kp; i += 256) yr[i] = fh_to<T>(0.f);
}

size_t fh_rec_chunk_floats(const FhRecurrent &, int) { return 0; }

fh_status fh_recurrent_prefill(fh_device *dev, int dtype, const FhRecurrent &r, const FhRecState &st, const float *proj,
                               int64_t ldp, int s, int pos, const FhRecWork &w, void *y, int kp) {
    hipStream_t str = dev->stream;
    const int nq = r.kv_heads * r.dim, inner = fh_rec_inner(r), channels = fh_rec_channels(r);
    const size_t lds1 = (size_t)2 * nq * 4, lds2 = (size_t)inner * 4;
    FH_REQUIRE(lds1 <= 150 * 1024 && lds2 <= 150 * 1024, "recurrent layer of %d channels is too wide", channels);
    if (lds1 > 48 * 1024) FH_TRY(fh_kernel_lds(dev, (const void *)k_rec_prep, lds1));
    k_rec_prep<<<dim3((unsigned)s), 256, lds1, str>>>(r, proj, ldp, pos, st.conv, w);
    const int ty = s < r.taps ? s : r.taps;
    k_rec_tail<<<dim3((unsigned)((channels + 255) / 256), (unsigned)ty), 256, 0, str>>>(r, proj, ldp, s, pos, st.conv);
    const dim3 sg((unsigned)((r.vdim + 3) / 4), (unsigned)r.heads);
    const int rpt = (r.dim + 15) / 16;
    if (rpt <= 2) k_rec_scan<2><<<sg, 64, 0, str>>>(r, w, st.s, s, pos == 0);
    else if (rpt <= 4) k_rec_scan<4><<<sg, 64, 0, str>>>(r, w, st.s, s, pos == 0);
    else if (rpt <= 8) k_rec_scan<8><<<sg, 64, 0, str>>>(r, w, st.s, s, pos == 0);
    else if (rpt <= 16) k_rec_scan<16><<<sg, 64, 0, str>>>(r, w, st.s, s, pos == 0);
    else FH_FAIL(FH_ERR_UNSUPPORTED, "recurrent state of %d rows (at most 256)", r.dim);
    if (dtype == FH_F32) {
        if (lds2 > 48 * 1024) FH_TRY(fh_kernel_lds(dev, (const void *)k_rec_out<float>, lds2));
        k_rec_out<float><<<dim3((unsigned)s), 256, lds2, str>>>(r, w.o, proj, ldp, (float *)y, kp);
    } else {
        if (lds2 > 48 * 1024) FH_TRY(fh_kernel_lds(dev, (const void *)k_rec_out<uint16_t>, lds2));
        k_rec_out<uint16_t><<<dim3((unsigned)s), 256, lds2, str>>>(r, w.o, proj, ldp, (uint16_t *)y, kp);
    }
    FH_HIP(hipGetLastError());
    return FH_OK;
}
