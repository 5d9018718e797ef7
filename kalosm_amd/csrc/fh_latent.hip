// Latent attention (fh_latent.h): cache rows, prefill on the matrix cores, decode step over the cached rows.
#include "fh_latent.h"

static constexpr float FH_LOG2E = 1.4426950408889634f;

// ------------------------------------------------------------------------------ cache rows of a portion
// Rows 0 .. old - 1 come out of the ring, the others are computed from the projections.  One workgroup per row.
template <typename T>
__global__ __launch_bounds__(128) void k_latent_rows(FhLatent a, const float *__restrict__ proj, int64_t ldp, int old, int pos,
                                                     const T *__restrict__ ring, int cap, T *__restrict__ lat, T *__restrict__ kr) {
    __shared__ float red[2];
    const int i = blockIdx.x, tid = threadIdx.x, row = a.r8 + a.drp;
    T *lr = lat + (int64_t)i * a.rp, *kd = kr + (int64_t)i * a.drp;
    if (i < old) {
        const T *src = ring + (int64_t)((pos - old + i) % cap) * row;
        for (int c = tid; c < a.rp; c += 128) lr[c] = c < a.r8 ? src[c] : fh_to<T>(0.f);
        for (int c = tid; c < a.drp; c += 128) kd[c] = src[a.r8 + c];
        return;
    }
    const int t = i - old;
    const float *p = proj + (int64_t)t * ldp + a.col_kv;
    float ss = 0.f;
    for (int c = tid; c < a.rank; c += 128) ss = fmaf(p[c], p[c], ss);
    ss = fh_wave_sum(ss);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();
    const float inv = 1.0f / sqrtf((red[0] + red[1]) / (float)a.rank + a.eps);
    for (int c = tid; c < a.rp; c += 128) lr[c] = fh_to<T>(c < a.rank ? p[c] * inv * a.c_norm[c] : 0.f);
    const float *ct = a.cos_t + (int64_t)(pos + t) * a.pairs, *st = a.sin_t + (int64_t)(pos + t) * a.pairs;
    for (int c = tid; c < a.drp; c += 128) {
        float v = c < a.dr ? p[a.rank + c] : 0.f;
        const int pr = c >> 1;
        if (c < a.dr && pr < a.pairs) {
            const float o = p[a.rank + (c ^ 1)];
            v = (c & 1) ? v * ct[pr] + o * st[pr] : v * ct[pr] - o * st[pr];
        }
        kd[c] = fh_to<T>(v);
    }
}

// The last `n` rows of the portion into the ring.
template <typename T>
__global__ __launch_bounds__(128) void k_latent_append(FhLatent a, const T *__restrict__ lat, const T *__restrict__ kr, int first,
                                                       int pos_first, T *__restrict__ ring, int cap) {
    const int i = blockIdx.x, row = a.r8 + a.drp;
    T *dst = ring + (int64_t)((pos_first + i) % cap) * row;
    for (int c = threadIdx.x; c < row; c += 128)
        dst[c] = c < a.r8 ? lat[(int64_t)(first + i) * a.rp + c] : kr[(int64_t)(first + i) * a.drp + c - a.r8];
}

// Queries [s, heads, dq]: unrotated part, rotated part, zeros.
template <typename T>
__global__ __launch_bounds__(256) void k_latent_q(FhLatent a, const float *__restrict__ proj, int64_t ldp, int pos, int dq,
                                                  T *__restrict__ q) {
    const int t = blockIdx.x, d0 = a.dn + a.dr;
    const float *p = proj + (int64_t)t * ldp + a.col_q;
    const float *ct = a.cos_t + (int64_t)(pos + t) * a.pairs, *st = a.sin_t + (int64_t)(pos + t) * a.pairs;
    for (int i = threadIdx.x; i < a.heads * dq; i += 256) {
        const int h = i / dq, c = i % dq;
        float v = 0.f;
        if (c < a.dn) v = p[h * d0 + c];
        else if (c >= a.dnp && c - a.dnp < a.dr) {
            const int r = c - a.dnp, pr = r >> 1;
            const float *pp = p + h * d0 + a.dn;
            v = pp[r];
            if (pr < a.pairs) {
                const float o = pp[r ^ 1];
                v = (r & 1) ? v * ct[pr] + o * st[pr] : v * ct[pr] - o * st[pr];
            }
        }
        q[((int64_t)t * a.heads + h) * dq + c] = fh_to<T>(v);
    }
}

int fh_latent_dq(const FhLatent &a) { return fh_window_dq(a.dnp + a.drp); }

template <typename T>
static fh_status latent_prefill_t(fh_device *dev, int dtype, const FhLatent &a, fh_kvcache *cache, const float *proj, int64_t ldp,
                                  int s, int pos, const FhLatentWork &w, void *o, int kp) {
    hipStream_t str = dev->stream;
    const int old = fh_latent_old(a, pos), keys = old + s, dq = fh_latent_dq(a);
    FH_REQUIRE(dq, "attention over %d + %d query dimensions (at most 256)", a.dn, a.dr);
    k_latent_rows<T><<<dim3((unsigned)keys), 128, 0, str>>>(a, proj, ldp, old, pos, (const T *)cache->k, cache->capacity, (T *)w.lat,
                                                           (T *)w.kr);
    const int n = s < cache->capacity ? s : cache->capacity;
    k_latent_append<T><<<dim3((unsigned)n), 128, 0, str>>>(a, (const T *)w.lat, (const T *)w.kr, keys - n, pos + s - n, (T *)cache->k,
                                                          cache->capacity);
    k_latent_q<T><<<dim3((unsigned)s), 256, 0, str>>>(a, proj, ldp, pos, dq, (T *)w.q);
    FH_HIP(hipGetLastError());
    FhGemm g;
    g.kp = a.rp, g.m = keys, g.x = w.lat;
    g.w = a.uk, g.n = a.heads * a.dnp, g.y = w.kn, g.ldy = (int64_t)a.heads * a.dnp;
    FH_TRY(fh_gemm(dev, dtype, FH_GEMM_ACT, g));
    g.w = a.uv, g.n = a.heads * a.dv, g.y = w.vt, g.ldy = w.ldt;
    FH_TRY(fh_gemm(dev, dtype, FH_GEMM_ACT_T, g));
    FhWindowAttn v;
    v.heads = a.heads, v.dnp = a.dnp, v.drp = a.drp, v.dv = a.dv, v.window = a.window, v.scale = a.scale, v.sink = a.sink;
    v.pos = pos, v.gap = pos - old;
    return fh_window_attn(dev, dtype, v, w.q, w.kn, w.kr, w.vt, w.ldt, s, keys, o, kp, kp);
}

fh_status fh_latent_prefill(fh_device *dev, int dtype, const FhLatent &a, fh_kvcache *cache, const float *proj, int64_t ldp,
                            int s, int pos, const FhLatentWork &w, void *o, int kp) {
    return dtype == FH_F32 ? latent_prefill_t<float>(dev, dtype, a, cache, proj, ldp, s, pos, w, o, kp)
                           : latent_prefill_t<uint16_t>(dev, dtype, a, cache, proj, ldp, s, pos, w, o, kp);
}

// ------------------------------------------------------------------------------ decode step
// grid (splits, head groups of HB).  The live rows of the ring are 0 .. min(position + 1, capacity) - 1 in any order (the
// softmax does not care, the rotation is already in the row).  The 16 lanes of a DPP row take one cached row, pieces of 8
// elements dealt round-robin; each row group keeps running statistics and a weighted sum of its own.
template <typename T, int NP, int HB> // NP pieces per lane: rows of at most 128 NP elements
__global__ __launch_bounds__(256) void k_latent_decode(FhLatent a, const T *__restrict__ ring, int cap, const int *__restrict__ pos_dev,
                                                       const float *__restrict__ qa, float *__restrict__ part) {
    extern __shared__ float od[]; // [4 waves][HB][r8 + 2]
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, l16 = lane & 15, rg = tid >> 4;
    const int row = a.r8 + a.drp, np = row / 8, h0 = (int)blockIdx.y * HB;
    const int n = *pos_dev + 1 < cap ? *pos_dev + 1 : cap;
    const int per = ((n + (int)gridDim.x - 1) / (int)gridDim.x + 15) / 16 * 16;
    const int k0 = (int)blockIdx.x * per, k1 = k0 + per < n ? k0 + per : n;
    float q[HB][NP][8], o[HB][NP][8], m[HB], l[HB];
#pragma unroll
    for (int b = 0; b < HB; b++) {
        m[b] = -INFINITY, l[b] = 0.f;
        const float *qp = qa + (int64_t)(h0 + b < a.heads ? h0 + b : a.heads - 1) * row;
#pragma unroll
        for (int i = 0; i < NP; i++)
#pragma unroll
            for (int e = 0; e < 8; e++) {
                q[b][i][e] = l16 + 16 * i < np ? qp[(l16 + 16 * i) * 8 + e] : 0.f;
                o[b][i][e] = 0.f;
            }
    }
    FhPiece<T> nx[NP];
    auto fetch = [&](int k) {
#pragma unroll
        for (int i = 0; i < NP; i++)
            nx[i] = l16 + 16 * i < np ? fh_ld_piece(ring + (int64_t)k * row + (l16 + 16 * i) * 8) : fh_zero_piece<T>();
    };
    if (k0 + rg < k1) fetch(k0 + rg);
    for (int k = k0 + rg; k < k1; k += 16) {
        float c[NP][8];
#pragma unroll
        for (int i = 0; i < NP; i++)
#pragma unroll
            for (int e = 0; e < 8; e++) c[i][e] = fh_up(nx[i].v[e]);
        if (k + 16 < k1) fetch(k + 16);
#pragma unroll
        for (int b = 0; b < HB; b++) {
            float d = 0.f;
#pragma unroll
            for (int i = 0; i < NP; i++)
#pragma unroll
                for (int e = 0; e < 8; e++) d = fmaf(q[b][i][e], c[i][e], d);
            d = fh_row16_sum(d);
            const float mn = fmaxf(m[b], d), r = exp2f(m[b] - mn), w = exp2f(d - mn);
            l[b] = l[b] * r + w;
            m[b] = mn;
#pragma unroll
            for (int i = 0; i < NP; i++)
#pragma unroll
                for (int e = 0; e < 8; e++) o[b][i][e] = fmaf(w, c[i][e], o[b][i][e] * r);
        }
    }
    const int st = a.r8 + 2;
#pragma unroll
    for (int b = 0; b < HB; b++) {
        // the four row groups of the wavefront, then the four wavefronts through the LDS
        float mm = fmaxf(m[b], __shfl_xor(m[b], 16, 64));
        mm = fmaxf(mm, __shfl_xor(mm, 32, 64));
        const float f = m[b] == -INFINITY ? 0.f : exp2f(m[b] - mm);
        float ll = l[b] * f;
        ll += __shfl_xor(ll, 16, 64);
        ll += __shfl_xor(ll, 32, 64);
        float *dst = od + (wave * HB + b) * st;
#pragma unroll
        for (int i = 0; i < NP; i++)
#pragma unroll
            for (int e = 0; e < 8; e++) {
                float v = o[b][i][e] * f;
                v += __shfl_xor(v, 16, 64);
                v += __shfl_xor(v, 32, 64);
                const int x = (l16 + 16 * i) * 8 + e;
                if (lane < 16 && x < a.r8) dst[x] = v;
            }
        if (lane == 0) dst[a.r8] = mm, dst[a.r8 + 1] = ll;
    }
    __syncthreads();
#pragma unroll
    for (int b = 0; b < HB; b++) {
        if (h0 + b >= a.heads) break;
        float mm = -INFINITY, f[4], ll = 0.f;
#pragma unroll
        for (int w = 0; w < 4; w++) mm = fmaxf(mm, od[(w * HB + b) * st + a.r8]);
#pragma unroll
        for (int w = 0; w < 4; w++) {
            const float mw = od[(w * HB + b) * st + a.r8];
            f[w] = mw == -INFINITY ? 0.f : exp2f(mw - mm);
            ll += f[w] * od[(w * HB + b) * st + a.r8 + 1];
        }
        float *dst = part + ((int64_t)(h0 + b) * gridDim.x + blockIdx.x) * st;
        for (int x = tid; x < a.r8; x += 256) {
            float v = 0.f;
#pragma unroll
            for (int w = 0; w < 4; w++) v = fmaf(f[w], od[(w * HB + b) * st + x], v);
            dst[x] = v;
        }
        if (tid == 0) dst[a.r8] = mm, dst[a.r8 + 1] = ll;
    }
}

// The same on the matrix cores, for bf16 caches: 16 heads are the rows of every product and a workgroup takes tiles of 64
// keys.  Scores (16 heads x 64 keys) = qa . C^T, one key block of 16 per wavefront, qa as hi + lo; softmax through the
// LDS, 16 lanes per head; sums (16 heads x rank) += P . C, P as hi + lo, a quarter of the rank per wavefront, the operand
// of C with the keys along k by the transposing LDS load (ds_read_b64_tr_b16: a lane receives its column of four rows).
typedef short fh_s4 __attribute__((ext_vector_type(4)));
__device__ __forceinline__ fh_bf8 lat_tr8(const uint16_t *p, int row_stride) { // rows k .. k + 3 and k + 16 .. k + 19
    const fh_s4 a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) fh_s4 *)(uintptr_t)(uint32_t)(uintptr_t)(__attribute__((address_space(3))) const void *)p);
    const fh_s4 b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) fh_s4 *)(uintptr_t)(uint32_t)(uintptr_t)(__attribute__((address_space(3))) const void *)(p + 16 * row_stride));
    fh_bf8 r;
    __builtin_memcpy(&r, &a, 8);
    __builtin_memcpy((char *)&r + 8, &b, 8);
    return r;
}

template <int NT> // 16-wide rank tiles of a wavefront: rank at most 64 NT
__global__ __launch_bounds__(256) void k_latent_decode_mfma(FhLatent a, const uint16_t *__restrict__ ring, int cap,
                                                            const int *__restrict__ pos_dev, const float *__restrict__ qa,
                                                            float *__restrict__ part) {
    extern __shared__ __attribute__((aligned(16))) char ld_lds[];
    const int row = a.r8 + a.drp, steps = (row + 95) / 96 * 3, CS = steps * 32 + 8; // steps of 32 (threes of them), LDS row stride
    uint16_t *sc = (uint16_t *)ld_lds, *sq = sc + 64 * CS, *sp = sq + 2 * 16 * CS; // cache tile, qa hi / lo, P hi / lo
    constexpr int PS = 72, SS = 68;
    float *s_s = (float *)(sp + 2 * 16 * PS), *s_r = s_s + 16 * SS; // scores, rescale factors
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, li = lane & 15, g = lane >> 4;
    const int h0 = (int)blockIdx.y * 16, np = row / 8, npp = steps * 4;
    const int n = *pos_dev + 1 < cap ? *pos_dev + 1 : cap;
    const int per = ((n + (int)gridDim.x - 1) / (int)gridDim.x + 15) / 16 * 16;
    const int k0 = (int)blockIdx.x * per, k1 = k0 + per < n ? k0 + per : n;
    auto stage = [&](int k) { // pieces of eight elements, four threads per row; zeros behind the row and behind the last key
        const int r = tid >> 2;
        const bool in = k + r < k1;
        const uint16_t *src = ring + (int64_t)(in ? k + r : 0) * row;
        for (int c0 = tid & 3; c0 < npp; c0 += 36) { // nine requests on their way at a time
            uint4 v[9];
#pragma unroll
            for (int j = 0; j < 9; j++) v[j] = in && c0 + 4 * j < np ? *(const uint4 *)(src + (c0 + 4 * j) * 8) : uint4{0, 0, 0, 0};
#pragma unroll
            for (int j = 0; j < 9; j++)
                if (c0 + 4 * j < npp) *(uint4 *)(sc + r * CS + (c0 + 4 * j) * 8) = v[j];
        }
    };
    {
        const int r = tid >> 4;
        const float *src = qa + (int64_t)(h0 + r < a.heads ? h0 + r : 0) * row;
        float4 x[5], y[5];
        auto get = [&](int c0) {
#pragma unroll
            for (int j = 0; j < 5; j++) {
                const int c = c0 + 16 * j;
                const bool in = c < np && h0 + r < a.heads;
                x[j] = in ? *(const float4 *)(src + c * 8) : make_float4(0.f, 0.f, 0.f, 0.f);
                y[j] = in ? *(const float4 *)(src + c * 8 + 4) : make_float4(0.f, 0.f, 0.f, 0.f);
            }
        };
        get(tid & 15);
        stage(k0);
        for (int c0 = tid & 15; c0 < npp; c0 += 80) {
            if (c0 >= 80) get(c0);
#pragma unroll
            for (int j = 0; j < 5; j++) {
                const int c = c0 + 16 * j;
                const float v[8] = {x[j].x, x[j].y, x[j].z, x[j].w, y[j].x, y[j].y, y[j].z, y[j].w};
                uint16_t hi[8], lo[8];
#pragma unroll
                for (int e = 0; e < 8; e++) hi[e] = fh_f32_bf(v[e]), lo[e] = fh_f32_bf(v[e] - fh_bf_f32(hi[e]));
                if (c < npp) {
                    __builtin_memcpy(sq + r * CS + c * 8, hi, 16);
                    __builtin_memcpy(sq + (16 + r) * CS + c * 8, lo, 16);
                }
            }
        }
    }
    fh_f4 o[NT];
#pragma unroll
    for (int t = 0; t < NT; t++) o[t] = fh_f4{0.f, 0.f, 0.f, 0.f};
    float mx = -INFINITY, den = 0.f; // of head tid / 16, the same in its 16 lanes
    for (int k = k0; k < k1; k += 64) {
        __syncthreads();
        fh_f4 S = fh_f4{0.f, 0.f, 0.f, 0.f};
        if (k + 16 * wave < k1)
            for (int x = 0; x < steps; x += 3) {
                fh_bf8 c[3], h[3], l[3];
#pragma unroll
                for (int j = 0; j < 3; j++) {
                    fh_frag_load(c[j], sc + (16 * wave + li) * CS + 32 * (x + j) + 8 * g);
                    fh_frag_load(h[j], sq + li * CS + 32 * (x + j) + 8 * g);
                    fh_frag_load(l[j], sq + (16 + li) * CS + 32 * (x + j) + 8 * g);
                }
#pragma unroll
                for (int j = 0; j < 3; j++) S = fh_mma32(h[j], c[j], S), S = fh_mma32(l[j], c[j], S);
            }
#pragma unroll
        for (int e = 0; e < 4; e++) s_s[(4 * g + e) * SS + 16 * wave + li] = k + 16 * wave + li < k1 ? S[e] : -INFINITY;
        __syncthreads();
        {
            const int hr = tid >> 4, kq = (tid & 15) * 4; // head row and four keys
            const float4 s4 = *(const float4 *)(s_s + hr * SS + kq);
            float tm = fmaxf(fmaxf(s4.x, s4.y), fmaxf(s4.z, s4.w));
#define FH_ROR(N_) tm = fmaxf(tm, __uint_as_float(__builtin_amdgcn_update_dpp(0, __float_as_uint(tm), 0x120 + N_, 0xF, 0xF, true)))
            FH_ROR(8);
            FH_ROR(4);
            FH_ROR(2);
            FH_ROR(1);
#undef FH_ROR
            const float mn = fmaxf(mx, tm), f = exp2f(mx - mn); // a tile has a live key, so mn is a number
            const float p[4] = {exp2f(s4.x - mn), exp2f(s4.y - mn), exp2f(s4.z - mn), exp2f(s4.w - mn)};
            den = den * f + fh_row16_sum((p[0] + p[1]) + (p[2] + p[3]));
            mx = mn;
            uint16_t hi[4], lo[4];
#pragma unroll
            for (int e = 0; e < 4; e++) hi[e] = fh_f32_bf(p[e]), lo[e] = fh_f32_bf(p[e] - fh_bf_f32(hi[e]));
            __builtin_memcpy(sp + hr * PS + kq, hi, 8);
            __builtin_memcpy(sp + (16 + hr) * PS + kq, lo, 8);
            if ((tid & 15) == 0) s_r[hr] = f;
        }
        __syncthreads();
        float f[4];
#pragma unroll
        for (int e = 0; e < 4; e++) f[e] = s_r[4 * g + e];
#pragma unroll
        for (int t = 0; t < NT; t++)
#pragma unroll
            for (int e = 0; e < 4; e++) o[t][e] *= f[e];
#pragma unroll
        for (int u = 0; u < 2; u++) {
            if (k + 32 * u >= k1) break;
            // k-slots of lane group g: keys 4 g .. + 3 and 16 + 4 g .. + 3, as the transposing load delivers them
            fh_bf8 ph, pl;
            __builtin_memcpy(&ph, sp + li * PS + 32 * u + 4 * g, 8);
            __builtin_memcpy((char *)&ph + 8, sp + li * PS + 32 * u + 16 + 4 * g, 8);
            __builtin_memcpy(&pl, sp + (16 + li) * PS + 32 * u + 4 * g, 8);
            __builtin_memcpy((char *)&pl + 8, sp + (16 + li) * PS + 32 * u + 16 + 4 * g, 8);
#pragma unroll
            for (int t = 0; t < NT; t++) {
                const int d = (wave * NT + t) * 16;
                if (d < a.r8) { // columns behind the rank (the rotated key, zeros) are never stored
                    const fh_bf8 c = lat_tr8(sc + (32 * u + 4 * g + (li >> 2)) * CS + d + (li & 3) * 4, CS);
                    o[t] = fh_mma32(ph, c, o[t]);
                    o[t] = fh_mma32(pl, c, o[t]);
                }
            }
        }
        __syncthreads();
        if (k + 64 < k1) stage(k + 64);
    }
    const int st = a.r8 + 2;
#pragma unroll
    for (int t = 0; t < NT; t++)
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int h = h0 + 4 * g + e, d = (wave * NT + t) * 16 + li;
            if (h < a.heads && d < a.r8) part[((int64_t)h * gridDim.x + blockIdx.x) * st + d] = o[t][e];
        }
    if ((tid & 15) == 0 && h0 + (tid >> 4) < a.heads) {
        float *p = part + ((int64_t)(h0 + (tid >> 4)) * gridDim.x + blockIdx.x) * st + a.r8;
        p[0] = mx, p[1] = den;
    }
}

// Merge of the splits (with the sink) and the value projection: grid (heads, blocks of 32 values).
__global__ __launch_bounds__(256) void k_latent_values(FhLatent a, const float *__restrict__ part, int splits, float *__restrict__ o,
                                                       const int *__restrict__ pos_dev, int cap) {
    extern __shared__ __attribute__((aligned(16))) float oc[]; // [rp]
    __shared__ float fw[FH_LATENT_MAX_SPLITS];
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, h = blockIdx.x, st = a.r8 + 2;
    const float *p = part + (int64_t)h * splits * st;
    const int n = *pos_dev + 1 < cap ? *pos_dev + 1 : cap, per = ((n + splits - 1) / splits + 15) / 16 * 16;
    const int live = (n + per - 1) / per; // splits that had keys
    uint4 w[8]; // the first 512 of k of this wavefront's rows, requested before the merge
    const int r0 = (int)blockIdx.y * 32 + wave * 8;
#pragma unroll
    for (int i = 0; i < 8; i++) {
        const int r = r0 + i < a.dv ? r0 + i : a.dv - 1;
        w[i] = lane * 8 < a.rp ? *(const uint4 *)(a.uv + (int64_t)(h * a.dv + r) * a.rp + lane * 8) : uint4{0, 0, 0, 0};
    }
    // this thread's two columns of the first 32 splits with keys
    auto two = [&](int i, int x) { return i < live && x < a.r8 ? *(const float2 *)(p + (int64_t)i * st + x) : make_float2(0.f, 0.f); };
    float2 y[32];
#pragma unroll
    for (int i = 0; i < 32; i++) y[i] = two(i, tid * 2);
    if (wave == 0) {
        static_assert(FH_LATENT_MAX_SPLITS <= 64, "one split per lane");
        const float z = a.sink ? a.sink[h] * FH_LOG2E : -INFINITY;
        const float m = lane < live ? p[lane * st + a.r8] : -INFINITY, l = lane < live ? p[lane * st + a.r8 + 1] : 0.f;
        float mm = fmaxf(m, z);
#pragma unroll
        for (int i = 32; i > 0; i >>= 1) mm = fmaxf(mm, __shfl_xor(mm, i, 64));
        const float f = m == -INFINITY ? 0.f : exp2f(m - mm);
        float d = fh_wave_sum(f * l);
        if (a.sink) d += exp2f(z - mm);
        fw[lane] = lane < live ? f / d : 0.f;
    }
    __syncthreads();
    for (int x = tid * 2; x < a.rp; x += 512) {
        float2 v = make_float2(0.f, 0.f);
        for (int i0 = 0; i0 < live; i0 += 32) {
            if (i0 || x >= 512)
#pragma unroll
                for (int i = 0; i < 32; i++) y[i] = two(i0 + i, x);
#pragma unroll
            for (int i = 0; i < 32; i++) v.x = fmaf(fw[i0 + i], y[i].x, v.x), v.y = fmaf(fw[i0 + i], y[i].y, v.y);
        }
        *(float2 *)(oc + x) = v;
    }
    __syncthreads();
    float acc[8];
#pragma unroll
    for (int i = 0; i < 8; i++) acc[i] = 0.f;
    for (int c = lane * 8; c < a.rp; c += 512) {
        const float4 x = *(const float4 *)(oc + c), y = *(const float4 *)(oc + c + 4);
#pragma unroll
        for (int i = 0; i < 8; i++) {
            const int r = r0 + i < a.dv ? r0 + i : a.dv - 1;
            const uint4 u = c < 512 ? w[i] : *(const uint4 *)(a.uv + (int64_t)(h * a.dv + r) * a.rp + c);
            acc[i] = fmaf(fh_bf_lo(u.x), x.x, acc[i]);
            acc[i] = fmaf(fh_bf_hi(u.x), x.y, acc[i]);
            acc[i] = fmaf(fh_bf_lo(u.y), x.z, acc[i]);
            acc[i] = fmaf(fh_bf_hi(u.y), x.w, acc[i]);
            acc[i] = fmaf(fh_bf_lo(u.z), y.x, acc[i]);
            acc[i] = fmaf(fh_bf_hi(u.z), y.y, acc[i]);
            acc[i] = fmaf(fh_bf_lo(u.w), y.z, acc[i]);
            acc[i] = fmaf(fh_bf_hi(u.w), y.w, acc[i]);
        }
    }
#pragma unroll
    for (int i = 0; i < 8; i++) acc[i] = fh_wave_sum(acc[i]);
    if (lane == 0)
#pragma unroll
        for (int i = 0; i < 8; i++)
            if (r0 + i < a.dv) o[h * a.dv + r0 + i] = acc[i];
}

template <typename T>
static fh_status latent_decode_t(fh_device *dev, const FhLatent &a, const fh_kvcache *cache, const int *pos_dev, const float *qa,
                                 float *part, float *o) {
    const int row = fh_latent_row(a), hb = a.heads % 2 == 0 ? 2 : 1;
    int splits = cache->capacity / 32;
    splits = splits < 1 ? 1 : splits > FH_LATENT_MAX_SPLITS ? FH_LATENT_MAX_SPLITS : splits;
    const int cs = (row + 95) / 96 * 96 + 8;
    const size_t mlds = (size_t)(96 * cs + 32 * 72) * 2 + (16 * 68 + 16) * 4;
    if (sizeof(T) == 2 && a.r8 <= 640 && mlds <= 156 * 1024 && dev->opt_attn_kernel != 1) {
        const dim3 mgrid((unsigned)splits, (unsigned)((a.heads + 15) / 16));
        const uint16_t *mring = (const uint16_t *)cache->k;
#define FH_GO(NT_)                                                                                                  \
    do {                                                                                                            \
        if (mlds > 48 * 1024) FH_TRY(fh_kernel_lds(dev, (const void *)k_latent_decode_mfma<NT_>, mlds));            \
        k_latent_decode_mfma<NT_><<<mgrid, 256, mlds, dev->stream>>>(a, mring, cache->capacity, pos_dev, qa, part); \
    } while (0)
        if (a.r8 <= 128) FH_GO(2);
        else if (a.r8 <= 512) FH_GO(8);
        else FH_GO(10);
#undef FH_GO
        k_latent_values<<<dim3((unsigned)a.heads, (unsigned)((a.dv + 31) / 32)), 256, (size_t)a.rp * 4, dev->stream>>>(a, part, splits, o, pos_dev, cache->capacity);
        FH_HIP(hipGetLastError());
        return FH_OK;
    }
    const dim3 grid((unsigned)splits, (unsigned)(a.heads / hb));
    const size_t lds = (size_t)4 * hb * (a.r8 + 2) * 4;
    const T *ring = (const T *)cache->k;
#define FH_GO(NP_)                                                                                                         \
    do {                                                                                                                   \
        if (lds > 48 * 1024) FH_TRY(fh_kernel_lds(dev, hb == 2 ? (const void *)k_latent_decode<T, NP_, 2> : (const void *)k_latent_decode<T, NP_, 1>, lds)); \
        if (hb == 2) k_latent_decode<T, NP_, 2><<<grid, 256, lds, dev->stream>>>(a, ring, cache->capacity, pos_dev, qa, part); \
        else k_latent_decode<T, NP_, 1><<<grid, 256, lds, dev->stream>>>(a, ring, cache->capacity, pos_dev, qa, part);     \
    } while (0)
    if (row <= 128) FH_GO(1);
    else if (row <= 256) FH_GO(2);
    else if (row <= 384) FH_GO(3);
    else if (row <= 640) FH_GO(5);
    else if (row <= 1152) FH_GO(9);
    else FH_FAIL(FH_ERR_UNSUPPORTED, "latent rows of %d elements (at most 1152)", row);
#undef FH_GO
    k_latent_values<<<dim3((unsigned)a.heads, (unsigned)((a.dv + 31) / 32)), 256, (size_t)a.rp * 4, dev->stream>>>(a, part, splits, o, pos_dev, cache->capacity);
    FH_HIP(hipGetLastError());
    return FH_OK;
}

fh_status fh_latent_decode(fh_device *dev, int dtype, const FhLatent &a, const fh_kvcache *cache, const int *pos_dev,
                           const float *qa, float *part, float *o) {
    return dtype == FH_F32 ? latent_decode_t<float>(dev, a, cache, pos_dev, qa, part, o)
                           : latent_decode_t<uint16_t>(dev, a, cache, pos_dev, qa, part, o);
}
