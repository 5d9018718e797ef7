// Prefill attention over a window (fh_window_attn.h).
#include "fh_window_attn.h"

static constexpr float FH_LOG2E = 1.4426950408889634f;

// grid (heads, query blocks, value blocks of 16 DVT): four wavefronts of 16 QF queries.  Both products are computed
// transposed, as in the other prefill attention: S^T = K . Q^T, O^T = V^T . P^T, so a lane (column) is one query and the
// softmax statistics are per-lane scalars.  MFMA row i of half hf of a 32-key group reads key 8 (i / 4) + 4 hf + i % 4:
// with that order the accumulators of a lane are keys 8 g .. 8 g + 7 (g = lane / 16), the k-slots of its P^T operand.
// Key tiles of 64 go through the LDS (K as [key][dq], V transposed as [value][key]); the next tile is requested into
// registers while the current one is multiplied.
// P^T operands: bf16 as hi + lo
__device__ __forceinline__ void fh_pv(fh_f4 &acc, const fh_bf8 &v, const float *p) {
    fh_bf8 hi, lo;
#pragma unroll
    for (int e = 0; e < 8; e++) {
        hi[e] = (fh_bf)p[e];
        lo[e] = (fh_bf)(p[e] - (float)hi[e]);
    }
    acc = fh_mma32(v, hi, acc);
    acc = fh_mma32(v, lo, acc);
}
__device__ __forceinline__ void fh_pv(fh_f4 &acc, const fh_f8 &v, const float *p) {
    fh_f8 b;
#pragma unroll
    for (int e = 0; e < 8; e++) b.v[e] = p[e];
    acc = fh_mma32(v, b, acc);
}

template <typename T, int DQS, int DVT, int QF>
__global__ __launch_bounds__(256) void k_window_attn(FhWindowAttn a, const T *__restrict__ q, const T *__restrict__ kn,
                                                     const T *__restrict__ kr, const T *__restrict__ vt, int64_t ldt, int s,
                                                     int keys, T *__restrict__ o, int ldo, int kp) {
    typedef typename FhFrag<T>::type Frag;
    constexpr int DQ = DQS * 32, KS = DQ + 8, VS = 64 + 8, QB = 64 * QF;
    constexpr int NK = 64 * DQ / 8 / 256, NV = DVT * 16 * 8 / 256; // pieces per thread
    static_assert(DVT % 2 == 0, "value pieces are shared out evenly");
    extern __shared__ __attribute__((aligned(16))) char wa_lds[];
    T *sk = (T *)wa_lds, *sv = sk + 64 * KS;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, li = lane & 15, g = lane >> 4;
    const int h = blockIdx.x, qb = (int)(gridDim.y - 1 - blockIdx.y) * QB, dv0 = (int)blockIdx.z * DVT * 16;
    const int npk = a.dnp / 8, nrk = a.drp / 8, hk = h / a.rep, kvh = a.heads / a.rep;
    Frag qf[DQS][QF];
    int qi[QF];
#pragma unroll
    for (int f = 0; f < QF; f++) {
        qi[f] = qb + wave * 16 * QF + f * 16 + li;
        const T *qp = q + ((int64_t)(qi[f] < s ? qi[f] : s - 1) * a.heads + h) * DQ + 8 * g;
#pragma unroll
        for (int k = 0; k < DQS; k++) fh_frag_load(qf[k][f], qp + 32 * k);
    }
    fh_f4 acc[DVT][QF];
    float mx[QF], den[QF];
#pragma unroll
    for (int f = 0; f < QF; f++) {
        mx[f] = -INFINITY, den[f] = 0.f;
#pragma unroll
        for (int d = 0; d < DVT; d++) acc[d][f] = fh_f4{0.f, 0.f, 0.f, 0.f};
    }
    const float sc = a.scale * FH_LOG2E;
    const int last = qb + QB - 1 < s ? qb + QB - 1 : s - 1;          // last query of the block
    // rows of the window of the block's first query, from its tile's start on; kept rows ahead of them are tiles of their own
    int j0 = a.window && a.pos + qb - a.window + 1 > 0 ? a.pos + qb - a.window + 1 : 0;
    if (j0 >= a.kept) j0 = j0 - a.gap > a.kept ? j0 - a.gap : a.kept;
    j0 = j0 / 64 * 64;
    const int j1 = a.pos + last - a.gap + 1;                         // one past the last visible key
    const int nk = a.keep < keys ? a.keep : keys;
    auto next = [&](int j) { return j + 64 >= nk && j + 64 < j0 ? j0 : j + 64; };
    FhPiece<T> pk[NK], pv[NV];
    auto fetch = [&](int j) {
#pragma unroll
        for (int i = 0; i < NK; i++) {
            const int x = tid + 256 * i, r = x / (DQ / 8), c = x % (DQ / 8);
            const int key = j + r;
            if (key < keys && c < npk) pk[i] = fh_ld_piece(kn + ((int64_t)key * kvh + hk) * a.dnp + c * 8);
            else if (key < keys && c - npk < nrk && c >= npk) pk[i] = fh_ld_piece(kr + (int64_t)key * a.drp + (c - npk) * 8);
            else pk[i] = fh_zero_piece<T>();
        }
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const int x = tid + 256 * i, r = x >> 3, c = (x & 7) * 8;
            if (dv0 + r < a.dv && j + c < keys) {
                pv[i] = fh_ld_piece(vt + (int64_t)(hk * a.dv + dv0 + r) * ldt + j + c);
                if (j + c + 8 > keys)
#pragma unroll
                    for (int e = 0; e < 8; e++)
                        if (j + c + e >= keys) pv[i].v[e] = 0;
            } else pv[i] = fh_zero_piece<T>();
        }
    };
    const int first = nk > 0 ? 0 : j0;
    fetch(first);
    for (int j = first; j < j1; j = next(j)) {
        __syncthreads(); // the previous tile has been read
#pragma unroll
        for (int i = 0; i < NK; i++) {
            const int x = tid + 256 * i, r = x / (DQ / 8), c = x % (DQ / 8);
            fh_st_piece(sk + r * KS + c * 8, pk[i]);
        }
#pragma unroll
        for (int i = 0; i < NV; i++) {
            const int x = tid + 256 * i, r = x >> 3, c = (x & 7) * 8;
            fh_st_piece(sv + r * VS + c, pv[i]);
        }
        __syncthreads();
        if (next(j) < j1) fetch(next(j));
        fh_f4 S[4][QF];
#pragma unroll
        for (int t = 0; t < 4; t++) {
#pragma unroll
            for (int f = 0; f < QF; f++) S[t][f] = fh_f4{0.f, 0.f, 0.f, 0.f};
            const T *kp_ = sk + (32 * (t >> 1) + 8 * (li >> 2) + 4 * (t & 1) + (li & 3)) * KS + 8 * g;
#pragma unroll
            for (int k = 0; k < DQS; k++) {
                Frag kf;
                fh_frag_load(kf, kp_ + 32 * k);
#pragma unroll
                for (int f = 0; f < QF; f++) S[t][f] = fh_mma32(kf, qf[k][f], S[t][f]);
            }
        }
        float p[QF][2][8];
#pragma unroll
        for (int f = 0; f < QF; f++) {
            float tm = -INFINITY;
#pragma unroll
            for (int t = 0; t < 4; t++)
#pragma unroll
                for (int r = 0; r < 4; r++) {
                    int kj = j + 32 * (t >> 1) + 8 * g + 4 * (t & 1) + r; // row, then position of the key
                    kj += kj >= a.kept ? a.gap : 0;
                    const int d = a.pos + qi[f] - kj;
                    const bool vis = d >= 0 && (!a.window || d < a.window || kj < a.keep);
                    const float v = vis ? S[t][f][r] * sc : -INFINITY;
                    p[f][t >> 1][4 * (t & 1) + r] = v;
                    tm = fmaxf(tm, v);
                }
            tm = fmaxf(tm, __shfl_xor(tm, 16, 64));
            tm = fmaxf(tm, __shfl_xor(tm, 32, 64));
            const float mn = fmaxf(mx[f], tm), mb = mn == -INFINITY ? 0.f : mn;
            const float resc = exp2f(mx[f] - mb);
            float sum = 0.f;
#pragma unroll
            for (int u = 0; u < 2; u++)
#pragma unroll
                for (int e = 0; e < 8; e++) {
                    const float w = exp2f(p[f][u][e] - mb);
                    p[f][u][e] = w;
                    sum += w;
                }
            den[f] = den[f] * resc + sum;
            mx[f] = mn;
#pragma unroll
            for (int d = 0; d < DVT; d++)
#pragma unroll
                for (int r = 0; r < 4; r++) acc[d][f][r] *= resc;
        }
#pragma unroll
        for (int u = 0; u < 2; u++)
#pragma unroll
            for (int d = 0; d < DVT; d++) {
                Frag vf;
                fh_frag_load(vf, sv + (16 * d + li) * VS + 32 * u + 8 * g);
#pragma unroll
                for (int f = 0; f < QF; f++) fh_pv(acc[d][f], vf, p[f][u]);
            }
    }
#pragma unroll
    for (int f = 0; f < QF; f++) {
        float l = den[f];
        l += __shfl_xor(l, 16, 64);
        l += __shfl_xor(l, 32, 64);
        if (qi[f] >= s) continue;
        float m = mx[f], up = 1.f;
        if (a.sink) { // the sink joins the denominator only
            const float z = a.sink[h] * FH_LOG2E, mm = fmaxf(m, z);
            up = exp2f(m - mm);
            l = l * up + exp2f(z - mm);
        }
        const float inv = up / l * a.out_scale;
        T *orow = o + (int64_t)qi[f] * ldo;
#pragma unroll
        for (int d = 0; d < DVT; d++)
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const int c = dv0 + 16 * d + 4 * g + r;
                if (c < a.dv) orow[h * a.dv + c] = fh_to<T>(acc[d][f][r] * inv);
            }
        if (h == a.heads - 1 && dv0 == 0)
            for (int c = a.heads * a.dv + g; c < kp; c += 4) orow[c] = fh_to<T>(0.f);
    }
}

int fh_window_dq(int dims) {
    const int d = (dims + 31) / 32;
    return d <= 2 ? 64 : d <= 4 ? 128 : d <= 6 ? 192 : d <= 8 ? 256 : 0;
}

template <typename T, int DQS, int DVT>
static fh_status window_attn_go(fh_device *dev, const FhWindowAttn &a, const void *q, const void *kn, const void *kr, const void *vt,
                                int64_t ldt, int s, int keys, void *o, int ldo, int kp) {
    constexpr int QF = sizeof(T) == 2 ? 2 : 1;
    const size_t lds = (size_t)(64 * (DQS * 32 + 8) + DVT * 16 * 72) * sizeof(T);
    auto fn = k_window_attn<T, DQS, DVT, QF>;
    if (lds > 48 * 1024) FH_TRY(fh_kernel_lds(dev, (const void *)fn, lds));
    const dim3 grid((unsigned)a.heads, (unsigned)((s + 64 * QF - 1) / (64 * QF)), (unsigned)((a.dv + DVT * 16 - 1) / (DVT * 16)));
    fn<<<grid, 256, lds, dev->stream>>>(a, (const T *)q, (const T *)kn, (const T *)kr, (const T *)vt, ldt, s, keys, (T *)o, ldo, kp);
    FH_HIP(hipGetLastError());
    return FH_OK;
}

template <typename T>
static fh_status window_attn_t(fh_device *dev, const FhWindowAttn &a, const void *q, const void *kn, const void *kr, const void *vt,
                               int64_t ldt, int s, int keys, void *o, int ldo, int kp) {
#define FH_GO(DQS_)                                                                                     \
    return a.dv <= 64 ? window_attn_go<T, DQS_, 4>(dev, a, q, kn, kr, vt, ldt, s, keys, o, ldo, kp)     \
                      : window_attn_go<T, DQS_, 8>(dev, a, q, kn, kr, vt, ldt, s, keys, o, ldo, kp)
    switch (fh_window_dq(a.dnp + a.drp)) {
    case 64: FH_GO(2);
    case 128: FH_GO(4);
    case 192: FH_GO(6);
    case 256: FH_GO(8);
    }
#undef FH_GO
    FH_FAIL(FH_ERR_UNSUPPORTED, "attention over %d query dimensions (at most 256)", a.dnp + a.drp);
}

fh_status fh_window_attn(fh_device *dev, int dtype, const FhWindowAttn &a, const void *q, const void *kn, const void *kr,
                         const void *vt, int64_t ldt, int s, int keys, void *o, int ldo, int kp) {
    return dtype == FH_F32 ? window_attn_t<float>(dev, a, q, kn, kr, vt, ldt, s, keys, o, ldo, kp)
                           : window_attn_t<uint16_t>(dev, a, q, kn, kr, vt, ldt, s, keys, o, ldo, kp);
}
