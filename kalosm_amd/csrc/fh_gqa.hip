// Prefill of grouped-query attention (fh_gqa.h): work rows of a portion, cache rows, and the windowed attention over them.
#include "fh_gqa.h"

// grid (s, groups of four heads): one wavefront per head - queries first, then keys, then values.
template <typename T, int J>
__global__ __launch_bounds__(256) void k_gqa_rows(FhGqa a, const float *__restrict__ proj, int64_t ldp, int old, int pos, int dq,
                                                  T *__restrict__ q, T *__restrict__ kn, T *__restrict__ vr) {
    __shared__ float tmp[4][64 * J], dst[4][64 * J];
    const int t = blockIdx.x, wave = threadIdx.x >> 6, lane = threadIdx.x & 63, job = (int)blockIdx.y * 4 + wave;
    const float *p = proj + (int64_t)t * ldp;
    const float *ct = a.cos_t + (int64_t)(pos + t) * a.pairs, *st = a.sin_t + (int64_t)(pos + t) * a.pairs;
    if (job < a.heads + a.kv_heads) {
        const bool key = job >= a.heads;
        const int h = key ? job - a.heads : job, pad = key ? a.dnp : dq;
        const float *norm = key ? a.k_norm : a.q_norm;
        FhHead<J> x;
        fh_head_load<J>(a, p + (key ? a.col_k : a.col_q) + h * a.dim, norm, ct, st, x);
        fh_head_rotate<J>(a, x, norm != nullptr, 1.f, tmp[wave], dst[wave]);
        T *o = key ? kn + ((int64_t)(old + t) * a.kv_heads + h) * a.dnp : q + ((int64_t)t * a.heads + h) * dq;
        for (int i = lane; i < pad; i += 64) o[i] = fh_to<T>(dst[wave][i]); // a lane reads back what it wrote
    } else if (job < a.heads + 2 * a.kv_heads) {
        const int h = job - a.heads - a.kv_heads;
        for (int i = lane; i < a.dvp; i += 64)
            vr[((int64_t)(old + t) * a.kv_heads + h) * a.dvp + i] = fh_to<T>(i < a.vdim ? p[a.col_v + h * a.vdim + i] : 0.f);
    }
}

// Rows ahead of the portion out of the cache.
template <typename T>
__global__ __launch_bounds__(256) void k_gqa_old(FhGqa a, const T *__restrict__ ring, int cap, int kept, int gap, T *__restrict__ kn,
                                                 T *__restrict__ vr) {
    const int j = blockIdx.x, nk = a.kv_heads * a.dnp, nv = a.kv_heads * a.dvp;
    const T *src = ring + (int64_t)fh_ring_row(j < kept ? j : j + gap, cap, a.keep) * (nk + nv);
    for (int i = threadIdx.x; i < nk; i += 256) kn[(int64_t)j * nk + i] = src[i];
    for (int i = threadIdx.x; i < nv; i += 256) vr[(int64_t)j * nv + i] = src[nk + i];
}

// The portion's rows that later positions may see, into the cache.
template <typename T>
__global__ __launch_bounds__(256) void k_gqa_append(FhGqa a, const T *__restrict__ kn, const T *__restrict__ vr, int old, int pos, int s,
                                                    T *__restrict__ ring, int cap) {
    const int t = blockIdx.x, p = pos + t, nk = a.kv_heads * a.dnp, nv = a.kv_heads * a.dvp;
    if (pos + s > cap && p >= a.keep && p < pos + s - (cap - a.keep)) return; // its row belongs to a later position
    T *dst = ring + (int64_t)fh_ring_row(p, cap, a.keep) * (nk + nv);
    for (int i = threadIdx.x; i < nk; i += 256) dst[i] = kn[(int64_t)(old + t) * nk + i];
    for (int i = threadIdx.x; i < nv; i += 256) dst[nk + i] = vr[(int64_t)(old + t) * nv + i];
}

// [keys, kv_heads * dvp] -> [kv_heads * vdim, ldt], tiles of 64 x 64.
template <typename T>
__global__ __launch_bounds__(256) void k_gqa_values(FhGqa a, const T *__restrict__ vr, int keys, T *__restrict__ vt, int64_t ldt) {
    __shared__ T tile[64][66];
    const int nv = a.kv_heads * a.dvp, j0 = (int)blockIdx.x * 64, c0 = (int)blockIdx.y * 64, lane = threadIdx.x & 63;
    for (int r = threadIdx.x >> 6; r < 64; r += 4)
        if (j0 + r < keys && c0 + lane < nv) tile[r][lane] = vr[(int64_t)(j0 + r) * nv + c0 + lane];
    __syncthreads();
    for (int r = threadIdx.x >> 6; r < 64; r += 4) {
        const int c = c0 + r, h = c / a.dvp, d = c % a.dvp;
        if (c < nv && d < a.vdim && j0 + lane < keys) vt[(int64_t)(h * a.vdim + d) * ldt + j0 + lane] = tile[lane][r];
    }
}

template <typename T>
static fh_status gqa_prefill_t(fh_device *dev, int dtype, const FhGqa &a, fh_kvcache *cache, const float *proj, int64_t ldp, int s, int pos,
                               const FhGqaWork &w, void *o, int ldo, int kp) {
    hipStream_t str = dev->stream;
    const int lo = fh_gqa_lo(a, pos), kept = fh_gqa_kept(a, pos), keys = fh_gqa_keys(a, s, pos), old = keys - s, dq = fh_window_dq(a.dnp);
    FH_REQUIRE(dq && w.ldt >= keys, "attention over %d query dimensions (at most 256)", a.dim);
    FH_REQUIRE(pos + s <= cache->capacity || cache->capacity == cache->max_len, "cache of %d rows has not grown to %d", cache->capacity, pos + s);
    T *q = (T *)w.q, *kn = (T *)w.kn, *vr = (T *)w.vr, *ring = (T *)cache->k;
    const dim3 rows((unsigned)s, (unsigned)((a.heads + 2 * a.kv_heads + 3) / 4));
    if (dq <= 128) k_gqa_rows<T, 2><<<rows, 256, 0, str>>>(a, proj, ldp, old, pos, dq, q, kn, vr);
    else k_gqa_rows<T, 4><<<rows, 256, 0, str>>>(a, proj, ldp, old, pos, dq, q, kn, vr);
    if (old > 0) k_gqa_old<T><<<dim3((unsigned)old), 256, 0, str>>>(a, ring, cache->capacity, kept, lo - kept, kn, vr);
    k_gqa_append<T><<<dim3((unsigned)s), 256, 0, str>>>(a, kn, vr, old, pos, s, ring, cache->capacity);
    k_gqa_values<T><<<dim3((unsigned)((keys + 63) / 64), (unsigned)((a.kv_heads * a.dvp + 63) / 64)), 256, 0, str>>>(a, vr, keys, (T *)w.vt, w.ldt);
    FH_HIP(hipGetLastError());
    FhWindowAttn v;
    v.heads = a.heads, v.rep = a.heads / a.kv_heads, v.dnp = a.dnp, v.dv = a.vdim, v.window = a.window, v.keep = a.window ? a.keep : 0;
    v.pos = pos, v.kept = kept, v.gap = lo - kept, v.scale = a.scale, v.out_scale = a.out_scale, v.sink = a.sink;
    return fh_window_attn(dev, dtype, v, w.q, w.kn, nullptr, w.vt, w.ldt, s, keys, o, ldo, kp);
}

fh_status fh_gqa_prefill(fh_device *dev, int dtype, const FhGqa &a, fh_kvcache *cache, const float *proj, int64_t ldp, int s, int pos,
                         const FhGqaWork &w, void *o, int ldo, int kp) {
    return dtype == FH_F32 ? gqa_prefill_t<float>(dev, dtype, a, cache, proj, ldp, s, pos, w, o, ldo, kp)
                           : gqa_prefill_t<uint16_t>(dev, dtype, a, cache, proj, ldp, s, pos, w, o, ldo, kp);
}
