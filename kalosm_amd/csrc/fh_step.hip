// Decode step kernels of the layer-list decoders (fh_step.h).
#include "fh_step.h"

static constexpr float FH_LOG2E = 1.4426950408889634f;

__device__ __forceinline__ float dot8(const uint4 &w, const float *x, float acc) {
    const float4 a = *(const float4 *)x, b = *(const float4 *)(x + 4);
    acc = fmaf(fh_bf_lo(w.x), a.x, acc);
    acc = fmaf(fh_bf_hi(w.x), a.y, acc);
    acc = fmaf(fh_bf_lo(w.y), a.z, acc);
    acc = fmaf(fh_bf_hi(w.y), a.w, acc);
    acc = fmaf(fh_bf_lo(w.z), b.x, acc);
    acc = fmaf(fh_bf_hi(w.z), b.y, acc);
    acc = fmaf(fh_bf_lo(w.w), b.z, acc);
    acc = fmaf(fh_bf_hi(w.w), b.w, acc);
    return acc;
}

// One step of a recurrence: workgroup b takes 16 columns of one head's state, RPT rows per lane as in the prefill scan.
template <int RPT>
__device__ __forceinline__ void rec_step(const FhStep &st, int b, float *lds) {
    const FhRecurrent &r = st.rec;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, rg = lane & 15;
    const int ncb = (r.vdim + 15) / 16, h = b / ncb, cb = b % ncb, d = r.dim, rep = r.heads / r.kv_heads, kh = h / rep;
    const int nq = r.kv_heads * d, channels = 2 * nq + r.heads * r.vdim, pos = *st.pos_dev;
    const int col = cb * 16 + wave * 4 + (lane >> 4), i0 = rg * RPT;
    const bool live = col < r.vdim;
    const int c = live ? col : r.vdim - 1;
    float *sp = st.rec_state.s + ((int64_t)h * r.vdim + c) * d;
    float S[RPT];
#pragma unroll
    for (int i = 0; i < RPT; i++) S[i] = pos > 0 && i0 + i < d ? sp[i0 + i] : 0.f;
    float *qk = lds, *vv = lds + 2 * d, *f = vv + 16; // [2 d], [16], [2]
    float *slot = st.rec_state.conv + (int64_t)(pos % r.taps) * channels; // not among the rows the convolution reads
    const bool keep = cb == 0 && h % rep == 0;        // one workgroup per key head stores its projections
    for (int i = tid; i < 2 * d; i += 256) {
        const int ch = i < d ? kh * d + i : nq + kh * d + i - d;
        qk[i] = fh_rec_conv(r, ch, st.proj, 0, 0, pos, st.rec_state.conv, channels);
        if (keep) slot[ch] = st.proj[i < d ? r.col_q + kh * d + i : r.col_k + kh * d + i - d];
    }
    if (tid < 16 && cb * 16 + tid < r.vdim) {
        const int vc = h * r.vdim + cb * 16 + tid;
        vv[tid] = fh_rec_conv(r, 2 * nq + vc, st.proj, 0, 0, pos, st.rec_state.conv, channels);
        slot[2 * nq + vc] = st.proj[r.col_v + vc];
    }
    __syncthreads();
    if (wave < 2) {
        float g = 1.f;
        if (r.delta()) {
            float ss = 0.f;
            for (int i = lane; i < d; i += 64) ss = fmaf(qk[wave * d + i], qk[wave * d + i], ss);
            g = 1.0f / sqrtf(fh_wave_sum(ss) + 1e-6f);
        }
        if (lane == 0) f[wave] = wave == 0 ? g * r.q_scale : g;
    }
    const float sp_ = fh_softplus_f(st.proj[r.col_a + h] + r.dt_bias[h]);
    const float g = expf(-expf(r.a_log[h]) * sp_), be = r.delta() ? fh_sigmoid_f(st.proj[r.col_b + h]) : sp_;
    __syncthreads();
    const float v = vv[live ? wave * 4 + (lane >> 4) : 0];
    float k[RPT], dot = 0.f, o = 0.f;
#pragma unroll
    for (int i = 0; i < RPT; i++) {
        k[i] = i0 + i < d ? qk[d + i0 + i] * f[1] : 0.f;
        S[i] *= g;
        dot = fmaf(S[i], k[i], dot);
    }
    const float u = r.delta() ? be * (v - fh_row16_sum(dot)) : be * v;
#pragma unroll
    for (int i = 0; i < RPT; i++) {
        S[i] = fmaf(k[i], u, S[i]);
        o = fmaf(S[i], i0 + i < d ? qk[i0 + i] * f[0] : 0.f, o);
        if (live && i0 + i < d) sp[i0 + i] = S[i];
    }
    o = fh_row16_sum(o);
    if (rg == 0 && live) st.o[h * r.vdim + col] = o + (r.d_skip ? r.d_skip[h] * v : 0.f);
}

// Absorbed queries of latent attention: workgroup b < heads * chunks takes 128 latent dimensions of one head, the last one
// appends this position's cache row.
template <typename T>
__device__ __forceinline__ void latent_step(const FhStep &st, T *ring, int cap, int b, float *lds) {
    const FhLatent &a = st.lat;
    const int tid = threadIdx.x, chunks = (a.r8 + 127) / 128, pos = *st.pos_dev, row = a.r8 + a.drp;
    const float *ct = a.cos_t + (int64_t)pos * a.pairs, *sn = a.sin_t + (int64_t)pos * a.pairs;
    if (b == a.heads * chunks) {
        const float *p = st.proj + a.col_kv;
        float ss = 0.f;
        for (int c = tid; c < a.rank; c += 256) ss = fmaf(p[c], p[c], ss);
        ss = fh_wave_sum(ss);
        if ((tid & 63) == 0) lds[tid >> 6] = ss;
        __syncthreads();
        const float inv = 1.0f / sqrtf((lds[0] + lds[1] + lds[2] + lds[3]) / (float)a.rank + a.eps);
        T *dst = ring + (int64_t)(pos % cap) * row;
        for (int c = tid; c < row; c += 256) {
            float v = 0.f;
            if (c < a.rank) v = p[c] * inv * a.c_norm[c];
            else if (c >= a.r8 && c - a.r8 < a.dr) {
                const int i = c - a.r8, pr = i >> 1;
                v = p[a.rank + i];
                if (pr < a.pairs) {
                    const float o = p[a.rank + (i ^ 1)];
                    v = (i & 1) ? v * ct[pr] + o * sn[pr] : v * ct[pr] - o * sn[pr];
                }
            }
            dst[c] = fh_to<T>(v);
        }
        return;
    }
    const int h = b / chunks, c0 = (b % chunks) * 128, sub = tid & 15, dg = tid >> 4, c = c0 + sub * 8;
    const float sc = a.scale * FH_LOG2E;
    const float *q = st.proj + a.col_q + h * (a.dn + a.dr);
    float acc[8];
#pragma unroll
    for (int e = 0; e < 8; e++) acc[e] = 0.f;
    if (c < a.rp)
        for (int d = dg; d < a.dn; d += 16) {
            const uint4 w = *(const uint4 *)(a.uk + (int64_t)(h * a.dnp + d) * a.rp + c);
            const float x = q[d];
            acc[0] = fmaf(fh_bf_lo(w.x), x, acc[0]);
            acc[1] = fmaf(fh_bf_hi(w.x), x, acc[1]);
            acc[2] = fmaf(fh_bf_lo(w.y), x, acc[2]);
            acc[3] = fmaf(fh_bf_hi(w.y), x, acc[3]);
            acc[4] = fmaf(fh_bf_lo(w.z), x, acc[4]);
            acc[5] = fmaf(fh_bf_hi(w.z), x, acc[5]);
            acc[6] = fmaf(fh_bf_lo(w.w), x, acc[6]);
            acc[7] = fmaf(fh_bf_hi(w.w), x, acc[7]);
        }
#pragma unroll
    for (int e = 0; e < 8; e++) lds[dg * 128 + sub * 8 + e] = acc[e];
    __syncthreads();
    float *dst = st.qa + (int64_t)h * row;
    if (tid < 128 && c0 + tid < a.r8) {
        float v = 0.f;
#pragma unroll
        for (int g = 0; g < 16; g++) v += lds[g * 128 + tid];
        dst[c0 + tid] = v * sc;
    }
    if (c0 == 0)
        for (int i = tid; i < a.drp; i += 256) {
            const int pr = i >> 1;
            float v = i < a.dr ? q[a.dn + i] : 0.f;
            if (i < a.dr && pr < a.pairs) {
                const float o = q[a.dn + (i ^ 1)];
                v = (i & 1) ? v * ct[pr] + o * sn[pr] : v * ct[pr] - o * sn[pr];
            }
            dst[a.r8 + i] = v * sc;
        }
}

// Gate and up products of the chosen experts: a workgroup takes 8 activations of one of them, two per wavefront.
__device__ __forceinline__ void expert_step(const FhStep &st, int b, float *lds) {
    const FhMoe &m = st.moe;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, tiles = (m.ff + 7) / 8, slot = b / tiles, tile = b % tiles;
    int *who = (int *)(lds + st.kp);
    if (wave == 0)
        fh_moe_route(st.proj + m.col_z, m.experts, m.scale, slot + 1, [&](int n, int e, float w) {
            if (n == slot && lane == 0) {
                *who = e;
                if (tile == 0) st.ids[slot] = e, st.wts[slot] = w;
            }
        });
    for (int i = tid * 4; i < st.kp; i += 1024) *(float4 *)(lds + i) = *(const float4 *)(st.hn + i);
    __syncthreads();
    const uint16_t *w = m.gate_up + (int64_t)*who * m.gu_stride;
    const uint16_t *row[4];
    const int p0 = tile * 8 + wave * 2;
#pragma unroll
    for (int i = 0; i < 2; i++) {
        const int p = p0 + i < m.ff ? p0 + i : m.ff - 1;
        row[2 * i] = w + (int64_t)(p / 16 * 32 + p % 16) * st.kp;
        row[2 * i + 1] = row[2 * i] + (int64_t)16 * st.kp;
    }
    float acc[4] = {0.f, 0.f, 0.f, 0.f};
    for (int c = lane * 8; c < st.kp; c += 512) {
        uint4 u[4];
#pragma unroll
        for (int i = 0; i < 4; i++) u[i] = *(const uint4 *)(row[i] + c);
#pragma unroll
        for (int i = 0; i < 4; i++) acc[i] = dot8(u[i], lds + c, acc[i]);
    }
#pragma unroll
    for (int i = 0; i < 4; i++) acc[i] = fh_wave_sum(acc[i]);
    if (lane == 0)
#pragma unroll
        for (int i = 0; i < 2; i++)
            if (p0 + i < m.ff) st.act[(int64_t)slot * m.ffp + p0 + i] = fh_silu_f(acc[2 * i]) * acc[2 * i + 1];
}

template <int RPT>
__global__ __launch_bounds__(256) void k_step_recurrent(FhStep st, int n_mix) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    if ((int)blockIdx.x < n_mix) rec_step<RPT>(st, blockIdx.x, lds);
    else expert_step(st, (int)blockIdx.x - n_mix, lds);
}
template <typename T>
__global__ __launch_bounds__(256) void k_step_latent(FhStep st, T *ring, int cap, int n_mix) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    if ((int)blockIdx.x < n_mix) latent_step<T>(st, ring, cap, blockIdx.x, lds);
    else expert_step(st, (int)blockIdx.x - n_mix, lds);
}

fh_status fh_step_middle(fh_device *dev, int dtype, const FhStep &st, fh_kvcache *cache) {
    const FhMoe &m = st.moe;
    const int n_exp = m.experts ? m.top * ((m.ff + 7) / 8) : 0;
    size_t lds = m.experts ? (size_t)(st.kp + 4) * 4 : 0;
    if (st.kind == FH_MIX_RECURRENT) {
        const int n_mix = st.rec.heads * ((st.rec.vdim + 15) / 16), rpt = (st.rec.dim + 15) / 16;
        const size_t need = (size_t)(2 * st.rec.dim + 32) * 4;
        lds = lds > need ? lds : need;
        const void *fn = rpt <= 2 ? (const void *)k_step_recurrent<2> : rpt <= 4 ? (const void *)k_step_recurrent<4>
                         : rpt <= 8 ? (const void *)k_step_recurrent<8> : (const void *)k_step_recurrent<16>;
        FH_REQUIRE(rpt <= 16, "recurrent state of %d rows (at most 256)", st.rec.dim);
        if (lds > 48 * 1024) FH_TRY(fh_kernel_lds(dev, fn, lds));
        const dim3 grid((unsigned)(n_mix + n_exp));
        if (rpt <= 2) k_step_recurrent<2><<<grid, 256, lds, dev->stream>>>(st, n_mix);
        else if (rpt <= 4) k_step_recurrent<4><<<grid, 256, lds, dev->stream>>>(st, n_mix);
        else if (rpt <= 8) k_step_recurrent<8><<<grid, 256, lds, dev->stream>>>(st, n_mix);
        else k_step_recurrent<16><<<grid, 256, lds, dev->stream>>>(st, n_mix);
    } else {
        const int n_mix = st.lat.heads * ((st.lat.r8 + 127) / 128) + 1;
        const size_t need = (size_t)16 * 128 * 4;
        lds = lds > need ? lds : need;
        const dim3 grid((unsigned)(n_mix + n_exp));
        if (lds > 48 * 1024)
            FH_TRY(fh_kernel_lds(dev, dtype == FH_F32 ? (const void *)k_step_latent<float> : (const void *)k_step_latent<uint16_t>, lds));
        if (dtype == FH_F32) k_step_latent<float><<<grid, 256, lds, dev->stream>>>(st, (float *)cache->k, cache->capacity, n_mix);
        else k_step_latent<uint16_t><<<grid, 256, lds, dev->stream>>>(st, (uint16_t *)cache->k, cache->capacity, n_mix);
    }
    FH_HIP(hipGetLastError());
    return FH_OK;
}

// ------------------------------------------------------------------------------ output launch
// One wavefront per row of the residual stream, eight rows per workgroup.  A row's weights - of the output projection, of
// the chosen experts and of the always-on one - are one list of pieces of 512; a table in the LDS says where each
// piece lies.  The first pieces are requested before the inputs are staged (the recurrent mixers' gate and norm are
// applied on the way into the LDS), later ones while earlier ones are multiplied.
struct OutPiece { const uint16_t *w; int kp, len, in; };
enum { FH_OUT_AHEAD = 8 };

__global__ __launch_bounds__(512) void k_step_out(FhStep st, int n_pieces) {
    extern __shared__ __attribute__((aligned(16))) float in[]; // [kpo | top * ffp | sffp | norm groups | pieces]
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const FhMoe &m = st.moe;
    const int n_e = m.experts ? m.top : 0, n_s = m.sff ? m.sffp : 0, n_in = st.kpo + n_e * m.ffp + n_s;
    const int n_g = st.kind == FH_MIX_RECURRENT ? (st.rec.norm_groups + 3) / 4 * 4 : 0;
    float *ie = in + st.kpo, *is = ie + n_e * m.ffp, *ginv = in + n_in;
    OutPiece *pt = (OutPiece *)(ginv + n_g);
    const int po = (st.kpo + 511) / 512, pe = (m.ffp + 511) / 512;
    for (int i = tid; i < n_pieces; i += 512) {
        OutPiece p;
        int k;
        if (i < po) k = i * 512, p.w = st.wo + k, p.kp = st.kpo, p.in = k;
        else if (i < po + n_e * pe) {
            const int j = (i - po) / pe;
            k = (i - po) % pe * 512;
            p.w = m.down + (int64_t)st.ids[j] * m.down_stride + k, p.kp = m.ffp, p.in = st.kpo + j * m.ffp + k;
        } else k = (i - po - n_e * pe) * 512, p.w = m.s_down + k, p.kp = m.sffp, p.in = st.kpo + n_e * m.ffp + k;
        p.len = p.kp - k;
        pt[i] = p;
    }
    __syncthreads();
    const int row = (int)blockIdx.x * 8 + wave, r = row < st.width ? row : st.width - 1;
    uint4 u[FH_OUT_AHEAD];
    auto fetch = [&](int i) -> uint4 {
        if (i >= n_pieces) return uint4{0, 0, 0, 0};
        const OutPiece p = pt[i];
        return lane * 8 < p.len ? *(const uint4 *)(p.w + (int64_t)r * p.kp + lane * 8) : uint4{0, 0, 0, 0};
    };
#pragma unroll
    for (int i = 0; i < FH_OUT_AHEAD; i++) u[i] = fetch(i);
    if (st.kind == FH_MIX_RECURRENT) {
        const FhRecurrent &rc = st.rec;
        const float *gate = st.proj + rc.col_g;
        const int inner = rc.heads * rc.vdim, gl = inner / rc.norm_groups;
        for (int i = tid; i < st.kpo; i += 512) {
            float v = i < inner ? st.o[i] : 0.f;
            if (rc.gate_first && i < inner) v *= fh_silu_f(gate[i]);
            in[i] = v;
        }
        __syncthreads();
        for (int g = wave; g < rc.norm_groups; g += 8) {
            float ss = 0.f;
            for (int i = lane; i < gl; i += 64) ss = fmaf(in[g * gl + i], in[g * gl + i], ss);
            ss = fh_wave_sum(ss);
            if (lane == 0) ginv[g] = 1.0f / sqrtf(ss / (float)gl + rc.eps);
        }
        __syncthreads();
        for (int i = tid; i < inner; i += 512) {
            float v = in[i] * ginv[i / gl] * rc.norm[rc.norm_len == inner ? i : i % rc.norm_len];
            if (!rc.gate_first) v *= fh_silu_f(gate[i]);
            in[i] = v;
        }
    } else {
        const int inner = st.lat.heads * st.lat.dv;
        for (int i = tid; i < st.kpo; i += 512) in[i] = i < inner ? st.o[i] : 0.f;
    }
#pragma unroll 4
    for (int i = tid * 4; i < n_e * m.ffp; i += 2048) {
        const int j = i / m.ffp, c = i % m.ffp;
        const float w = st.wts[j];
        const float4 v = *(const float4 *)(st.act + i);
        *(float4 *)(ie + i) = make_float4(c < m.ff ? w * v.x : 0.f, c + 1 < m.ff ? w * v.y : 0.f, c + 2 < m.ff ? w * v.z : 0.f,
                                          c + 3 < m.ff ? w * v.w : 0.f);
    }
    for (int i = tid; i < n_s; i += 512) {
        const int g = i / 16 * 32 + i % 16;
        is[i] = fh_silu_f(st.s_gu[g]) * st.s_gu[g + 16];
    }
    __syncthreads();
    float acc = 0.f;
    for (int b = 0; b < n_pieces; b += FH_OUT_AHEAD) {
#pragma unroll
        for (int i = 0; i < FH_OUT_AHEAD; i++) {
            const uint4 w = u[i];
            u[i] = fetch(b + i + FH_OUT_AHEAD);
            if (b + i < n_pieces && lane * 8 < pt[b + i].len) acc = dot8(w, in + pt[b + i].in + lane * 8, acc);
        }
    }
    acc = fh_wave_sum(acc);
    if (lane == 0 && row < st.width) st.x[row] += acc;
}

fh_status fh_step_out(fh_device *dev, const FhStep &st) {
    const FhMoe &m = st.moe;
    const int n_e = m.experts ? m.top : 0, n_s = m.sff ? m.sffp : 0;
    const int pieces = (st.kpo + 511) / 512 + n_e * ((m.ffp + 511) / 512) + (n_s + 511) / 512;
    const size_t lds = (size_t)(st.kpo + n_e * m.ffp + n_s + (st.kind == FH_MIX_RECURRENT ? (st.rec.norm_groups + 3) / 4 * 4 : 0)) * 4 +
                       (size_t)pieces * sizeof(OutPiece);
    FH_REQUIRE(lds <= 156 * 1024, "a decode step stages at most 156 KB of inputs (%zu bytes needed)", lds);
    if (lds > 48 * 1024) FH_TRY(fh_kernel_lds(dev, (const void *)k_step_out, lds));
    k_step_out<<<dim3((unsigned)((st.width + 7) / 8)), 512, lds, dev->stream>>>(st, pieces);
    FH_HIP(hipGetLastError());
    return FH_OK;
}

// ------------------------------------------------------------------------------ mixers of sublayers normed at their end
// RPT consecutive values from i0 on, those past d repeat the last one.
template <int RPT>
__device__ __forceinline__ void rec_load(float *v, const float *p, int i0, int d, bool full) {
    constexpr int N = RPT < 4 ? RPT : 4;
    if (full) {
#pragma unroll
        for (int i = 0; i < RPT; i += N) __builtin_memcpy(v + i, p + i0 + i, N * 4);
    } else {
#pragma unroll
        for (int i = 0; i < RPT; i++) v[i] = p[i0 + i < d ? i0 + i : d - 1];
    }
}

// One step of a recurrence without a short convolution: workgroup b takes 16 columns of one head's state.
template <int RPT>
__device__ __forceinline__ void linear_step(const FhMixStep &st, int pos, int b, float *lds) {
    const FhRecurrent &r = st.r;
    const int tid = threadIdx.x, lane = tid & 63, rg = lane & 15, d = r.dim;
    const int ncb = (r.vdim + 15) / 16, h = b / ncb, col = b % ncb * 16 + (tid >> 4), i0 = rg * RPT;
    const bool live = col < r.vdim;
    float *sp = st.state.s + ((int64_t)h * r.vdim + (live ? col : r.vdim - 1)) * d;
    float S[RPT];
    const bool full = d == 16 * RPT; // whole rows in float4s
    rec_load<RPT>(S, sp, i0, d, full);
#pragma unroll
    for (int i = 0; i < RPT; i++) S[i] = pos > 0 ? S[i] : 0.f;
    const float *q = st.proj + r.col_q + h * d, *k = st.proj + r.col_k + h * d;
    const float v = st.proj[r.col_v + h * r.vdim + (live ? col : r.vdim - 1)];
    float o = 0.f;
    if (r.kind == FH_REC_CHANNEL) {
        float *g = lds, *t1 = lds + 256; // [d], [rp]
        // every request goes out before the first wait
        uint4 w2[RPT];
        float kk[RPT], qq[RPT], uu[RPT], w0[RPT];
#pragma unroll
        for (int i = 0; i < RPT; i++) { // the 16 lanes of a DPP row share a channel: 16 i + tid / 16
            const int c = 16 * i + (tid >> 4);
            const int64_t cc = h * d + (c < d ? c : d - 1);
            w2[i] = *(const uint4 *)(r.w2 + cc * r.rp + (rg * 8 < r.rp ? rg * 8 : 0));
            w0[i] = r.w0[cc];
        }
        rec_load<RPT>(kk, k, i0, d, full);
        rec_load<RPT>(qq, q, i0, d, full);
        rec_load<RPT>(uu, r.bonus + h * d, i0, d, full);
#pragma unroll
        for (int i = 0; i < RPT; i++) // rows past the end read nothing out
            if (i0 + i >= d) kk[i] = 0.f, qq[i] = 0.f;
        for (int i = tid; i < r.rp; i += 256) t1[i] = i < r.rank ? st.proj[r.col_a + i] : 0.f;
        __syncthreads();
#pragma unroll
        for (int i = 0; i < RPT; i++) {
            const int c = 16 * i + (tid >> 4);
            float z = rg * 8 < r.rp ? dot8(w2[i], t1 + rg * 8, 0.f) : 0.f;
            if (c < d)
                for (int x = rg * 8 + 128; x < r.rp; x += 128) z = dot8(*(const uint4 *)(r.w2 + (int64_t)(h * d + c) * r.rp + x), t1 + x, z);
            z = fh_row16_sum(z);
            if (rg == 0 && c < d) g[c] = expf(fh_rec_la(z + w0[i]));
        }
        __syncthreads();
#pragma unroll
        for (int i = 0; i < RPT; i++) {
            const float kv = kk[i] * v;
            o = fmaf(fmaf(uu[i], kv, S[i]), qq[i], o);
            S[i] = fmaf(S[i], g[i0 + i], kv);
        }
    } else {
        const float g = expf(r.log_decay[h]), *ct = r.cos_t + (int64_t)pos * r.pairs, *sn = r.sin_t + (int64_t)pos * r.pairs;
        float *qk = lds; // [2][16 RPT], zeros from d on
        for (int i = tid; i < 32 * RPT; i += 256) {
            const bool key = i >= 16 * RPT;
            const int c0 = i % (16 * RPT), c = c0 < d ? c0 : d - 1, p = r.halves ? c < r.pairs ? c : c - r.pairs : c >> 1;
            const bool second = r.halves ? c >= r.pairs : c & 1, turn = c < 2 * r.pairs;
            const float *x = key ? k : q;
            const float y = x[c], z = x[!turn ? c : !r.halves ? c ^ 1 : second ? c - r.pairs : c + r.pairs];
            const float co = ct[turn ? p : 0], si = sn[turn ? p : 0];
            qk[i] = c0 < d ? (turn ? y * co + (second ? z * si : -z * si) : y) * (key ? r.k_scale : r.q_scale) : 0.f;
        }
        __syncthreads();
#pragma unroll
        for (int i = 0; i < RPT; i++) {
            S[i] = fmaf(qk[16 * RPT + i0 + i], v, S[i] * g);
            o = fmaf(S[i], qk[i0 + i], o);
        }
    }
    o = fh_row16_sum(o);
    if (!live) return;
    if (full)
#pragma unroll
        for (int i = 0; i < RPT; i += RPT < 4 ? RPT : 4) __builtin_memcpy(sp + i0 + i, S + i, (RPT < 4 ? RPT : 4) * 4);
    else
        for (int i = 0; i < RPT; i++)
            if (i0 + i < d) sp[i0 + i] = S[i];
    if (rg == 0) st.o[h * r.vdim + col] = o;
}

template <typename T, int NP, int RPT>
__global__ __launch_bounds__(256) void k_step_mixers(FhMixStep st, T *ring, int cap, int splits, int n_attn) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int pos = *st.pos_dev;
    if ((int)blockIdx.x < n_attn) fh_gqa_step<T, NP>(st.gqa, st.proj, ring, cap, pos, splits, blockIdx.x, st.part, lds);
    else linear_step<RPT>(st, pos, (int)blockIdx.x - n_attn, lds);
}

template <typename T, int NP>
static fh_status step_mixers_t(fh_device *dev, const FhMixStep &st, fh_kvcache *cache) {
    const int splits = st.attn ? fh_gqa_splits(cache) : 1, n_attn = st.attn ? fh_gqa_blocks(st.gqa, splits) : 0;
    const int n_rec = st.rec ? st.r.heads * ((st.r.vdim + 15) / 16) : 0, rpt = st.rec ? (st.r.dim + 15) / 16 : 1;
    size_t lds = st.attn ? fh_gqa_lds(st.gqa) : 0;
    const size_t need = !st.rec ? 0 : (size_t)(st.r.kind == FH_REC_CHANNEL ? 256 + st.r.rp : 512) * 4;
    lds = lds > need ? lds : need;
    FH_REQUIRE(lds <= 60 * 1024 && rpt <= 16, "mixers too wide for a decode step (%zu bytes of LDS)", lds);
    const dim3 grid((unsigned)(n_attn + n_rec));
    T *ring = cache ? (T *)cache->k : nullptr;
    const int cap = cache ? cache->capacity : 1;
    if (rpt <= 2) k_step_mixers<T, NP, 2><<<grid, 256, lds, dev->stream>>>(st, ring, cap, splits, n_attn);
    else if (rpt <= 4) k_step_mixers<T, NP, 4><<<grid, 256, lds, dev->stream>>>(st, ring, cap, splits, n_attn);
    else if (rpt <= 8) k_step_mixers<T, NP, 8><<<grid, 256, lds, dev->stream>>>(st, ring, cap, splits, n_attn);
    else k_step_mixers<T, NP, 16><<<grid, 256, lds, dev->stream>>>(st, ring, cap, splits, n_attn);
    FH_HIP(hipGetLastError());
    return FH_OK;
}

fh_status fh_step_mixers(fh_device *dev, int dtype, const FhMixStep &st, fh_kvcache *cache) {
    FH_REQUIRE(!st.attn || (cache && st.gqa.dnp <= 256 && st.gqa.dvp <= 256), "attention heads of a decode step have at most 256 dimensions");
    const bool one = !st.attn || (st.gqa.dnp <= 128 && st.gqa.dvp <= 128);
    if (dtype == FH_F32) return one ? step_mixers_t<float, 1>(dev, st, cache) : step_mixers_t<float, 2>(dev, st, cache);
    return one ? step_mixers_t<uint16_t, 1>(dev, st, cache) : step_mixers_t<uint16_t, 2>(dev, st, cache);
}

// One wavefront per attention head, then one per norm group of the recurrence.
__global__ __launch_bounds__(64) void k_step_mix_out(FhMixStep st, int splits) {
    const int lane = threadIdx.x, na = st.attn ? st.gqa.heads : 0, b = blockIdx.x;
    if (b < na) {
        const FhGqa &a = st.gqa;
        fh_gqa_merge(a, st.part, splits, b, st.act + b * a.vdim);
        if (b == na - 1)
            for (int i = a.heads * a.vdim + lane; i < st.kpl; i += 64) st.act[i] = 0.f;
        return;
    }
    const FhRecurrent &r = st.r;
    const int g = b - na, inner = r.heads * r.vdim, gl = inner / r.norm_groups;
    const float *o = st.o + g * gl, *gate = st.proj + r.col_g + g * gl;
    float ss = 0.f;
    for (int i = lane; i < gl; i += 64) ss = fmaf(o[i], o[i], ss);
    const float inv = 1.0f / sqrtf(fh_wave_sum(ss) / (float)gl + r.eps);
    for (int i = lane; i < gl; i += 64) {
        float v = o[i] * inv;
        if (r.norm) v *= r.norm[r.norm_len == inner ? g * gl + i : i % r.norm_len];
        st.act[st.kpl + g * gl + i] = v * fh_silu_f(gate[i]) * r.out_scale;
    }
}

fh_status fh_step_mix_out(fh_device *dev, const FhMixStep &st, const fh_kvcache *cache) {
    FH_REQUIRE(!st.rec || !st.r.gate_first, "this step gates behind the norm");
    const int blocks = (st.attn ? st.gqa.heads : 0) + (st.rec ? st.r.norm_groups : 0);
    k_step_mix_out<<<dim3((unsigned)blocks), 64, 0, dev->stream>>>(st, st.attn ? fh_gqa_splits(cache) : 1);
    FH_HIP(hipGetLastError());
    return FH_OK;
}
