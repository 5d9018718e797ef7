// Dense bf16 weights: prefill products on the matrix cores (plain and grouped by expert), the decode matvec with the
// RMS norm of its input, and the norm that writes activation rows.
#include "fh_dense.h"

// ------------------------------------------------------------------------------ prefill product
// y[m, n] = x[m, :] . W[n, :].  The weights are the A operand (accumulator rows), the activations the B operand
// (accumulator columns), so a lane holds four neighbouring outputs of one activation row; for the transposed output the
// operands change places and a lane holds four neighbouring activation rows of one output.
//
// bf16: 128 weight rows x BM activation rows per workgroup, four wavefronts, 64 of k per step.  Both operands go from
// memory straight into the LDS (LDS-direct loads, double buffered, one barrier per step).  An LDS row is 128 bytes =
// eight 16-byte pieces; piece c of row r sits at position c ^ ((r / 2) % 8), so that the 16 rows an operand read touches
// at one c cover the 64 banks once.  The swizzle is applied on the memory side of the loads.
template <int EPI, typename T>
__device__ __forceinline__ void gemm_store(void *y, int64_t ldy, int m_row, int n_row, const fh_f4 &v, int m, int n) {
    // EPI F32 / ACT: outputs n_row .. n_row + 3 of row m_row.  ACT_T: rows m_row .. m_row + 3 of output n_row.
    if (EPI == FH_GEMM_ACT_T) {
        if (n_row >= n) return;
        T *p = (T *)y + (int64_t)n_row * ldy + m_row;
#pragma unroll
        for (int r = 0; r < 4; r++)
            if (m_row + r < m) p[r] = fh_to<T>(v[r]);
        return;
    }
    if (m_row >= m) return;
    if (EPI == FH_GEMM_F32) {
        float *p = (float *)y + (int64_t)m_row * ldy + n_row;
        if (n_row + 3 < n && (ldy & 3) == 0) *(float4 *)p = make_float4(v[0], v[1], v[2], v[3]);
        else
#pragma unroll
            for (int r = 0; r < 4; r++)
                if (n_row + r < n) p[r] = v[r];
    } else {
        T *p = (T *)y + (int64_t)m_row * ldy + n_row;
        T t[4];
#pragma unroll
        for (int r = 0; r < 4; r++) t[r] = fh_to<T>(v[r]);
        if (n_row + 3 < n && (ldy & 3) == 0) {
            struct alignas(4 * sizeof(T)) V4 { T t[4]; };
            *(V4 *)p = V4{{t[0], t[1], t[2], t[3]}};
        } else
#pragma unroll
            for (int r = 0; r < 4; r++)
                if (n_row + r < n) p[r] = t[r];
    }
}

__device__ __forceinline__ fh_f4 relu2(fh_f4 v) {
#pragma unroll
    for (int e = 0; e < 4; e++) v[e] = fmaxf(v[e], 0.f) * fmaxf(v[e], 0.f);
    return v;
}

__device__ __forceinline__ int gemm_sw(int row) { return (row >> 1) & 7; }

template <int BM, int EPI>
__global__ __launch_bounds__(256) void k_gemm_bf16(FhGemm g) {
    constexpr int BN = 128, LDK = 64;
    constexpr int WM = BM >= 128 ? 2 : 1, WN = 4 / WM;        // wavefronts along m and n
    constexpr int FN = BN / WN / 16, FM = BM / WM / 16;       // 16 x 16 tiles of a wavefront
    constexpr int BUF = (BN + BM) * LDK;
    __shared__ __attribute__((aligned(16))) uint16_t smem[2 * BUF];
    const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63;
    const int wn = wave / WM, wm = wave % WM, li = lane & 15, gq = lane >> 4;
    int row0, m_end;
    const uint16_t *w = g.w;
    if (g.tiles) {
        if ((int)blockIdx.y >= *g.n_tiles) return;
        const FhTile t = g.tiles[blockIdx.y];
        row0 = t.row0;
        m_end = t.row0 + t.rows;
        w += (int64_t)t.group * g.w_group;
    } else {
        row0 = (int)blockIdx.y * BM;
        m_end = g.m;
    }
    const int n0 = (int)blockIdx.x * BN;
    const uint16_t *x = (const uint16_t *)g.x;
    // LDS-direct loads: a wavefront's request fills eight rows; lane l supplies row l / 8, position l % 8
    constexpr int NL_W = BN / 32, NL_X = BM / 32;
    const uint16_t *wp[NL_W], *xp[NL_X];
    const int rl = tid >> 3, pos = tid & 7;
#pragma unroll
    for (int i = 0; i < NL_W; i++) {
        const int r = rl + 32 * i, n = n0 + r < g.n ? n0 + r : g.n - 1; // rows past the end repeat the last one, never stored
        wp[i] = w + (int64_t)n * g.kp + (pos ^ gemm_sw(r)) * 8;
    }
#pragma unroll
    for (int i = 0; i < NL_X; i++) {
        const int r = rl + 32 * i;
        int m = row0 + r < m_end ? row0 + r : m_end - 1;
        if (g.gather) m = g.gather[m];
        xp[i] = x + (int64_t)m * g.kp + (pos ^ gemm_sw(r)) * 8;
    }
    auto fetch = [&](int ks) {
        uint16_t *dst = smem + (ks & 1) * BUF + wave * 8 * LDK;
#pragma unroll
        for (int i = 0; i < NL_W; i++)
            __builtin_amdgcn_global_load_lds((const uint32_t *)(wp[i] + ks * 64),
                                             (__attribute__((address_space(3))) uint32_t *)(dst + i * 32 * LDK), 16, 0, 0);
#pragma unroll
        for (int i = 0; i < NL_X; i++)
            __builtin_amdgcn_global_load_lds((const uint32_t *)(xp[i] + ks * 64),
                                             (__attribute__((address_space(3))) uint32_t *)(dst + (BN + i * 32) * LDK), 16, 0, 0);
    };
    fh_f4 acc[FN][FM];
#pragma unroll
    for (int a = 0; a < FN; a++)
#pragma unroll
        for (int b = 0; b < FM; b++) acc[a][b] = fh_f4{0.f, 0.f, 0.f, 0.f};
    const int steps = g.kp / 64;
    fetch(0);
    for (int ks = 0; ks < steps; ks++) {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory"); // this wavefront's pieces of step ks have landed
        __syncthreads();                                  // everybody's have, and nobody reads the other buffer any more
        if (ks + 1 < steps) fetch(ks + 1);
        const uint16_t *bw = smem + (ks & 1) * BUF, *bx = bw + BN * LDK;
#pragma unroll
        for (int kk = 0; kk < 2; kk++) {
            fh_bf8 fw[FN], fx[FM];
#pragma unroll
            for (int a = 0; a < FN; a++) {
                const int r = wn * FN * 16 + a * 16 + li;
                fh_frag_load(fw[a], bw + r * LDK + ((kk * 4 + gq) ^ gemm_sw(r)) * 8);
            }
#pragma unroll
            for (int b = 0; b < FM; b++) {
                const int r = wm * FM * 16 + b * 16 + li;
                fh_frag_load(fx[b], bx + r * LDK + ((kk * 4 + gq) ^ gemm_sw(r)) * 8);
            }
#pragma unroll
            for (int a = 0; a < FN; a++)
#pragma unroll
                for (int b = 0; b < FM; b++)
                    acc[a][b] = EPI == FH_GEMM_ACT_T ? fh_mma32(fx[b], fw[a], acc[a][b]) : fh_mma32(fw[a], fx[b], acc[a][b]);
        }
    }
#pragma unroll
    for (int b = 0; b < FM; b++) {
#pragma unroll
        for (int a = 0; a < FN; a += EPI == FH_GEMM_SWIGLU ? 2 : 1) {
            const int nb = n0 + wn * FN * 16 + a * 16, mb = row0 + wm * FM * 16 + b * 16;
            if (EPI == FH_GEMM_SWIGLU) {
                fh_f4 v;
#pragma unroll
                for (int r = 0; r < 4; r++) v[r] = fh_silu_f(acc[a][b][r]) * acc[a + 1 < FN ? a + 1 : a][b][r];
                gemm_store<FH_GEMM_ACT, uint16_t>(g.y, g.ldy, mb + li, nb / 2 + gq * 4, v, m_end, g.n / 2);
            } else if (EPI == FH_GEMM_RELU2) {
                gemm_store<FH_GEMM_ACT, uint16_t>(g.y, g.ldy, mb + li, nb + gq * 4, relu2(acc[a][b]), m_end, g.n);
            } else if (EPI == FH_GEMM_ACT_T) {
                gemm_store<EPI, uint16_t>(g.y, g.ldy, mb + gq * 4, nb + li, acc[a][b], m_end, g.n);
            } else {
                gemm_store<EPI, uint16_t>(g.y, g.ldy, mb + li, nb + gq * 4, acc[a][b], m_end, g.n);
            }
        }
    }
}

// f32 activations: 64 x 64 outputs per workgroup, 32 of k per step, true f32 products (v_mfma_f32_16x16x4_f32) of the
// widened weights.
template <int EPI>
__global__ __launch_bounds__(256) void k_gemm_f32(FhGemm g) {
    constexpr int BN = 64, BM = 64, LD = 36;
    __shared__ __attribute__((aligned(16))) float sw_[BN * LD], sx_[BM * LD];
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, wn = wave >> 1, wm = wave & 1, li = lane & 15, gq = lane >> 4;
    int row0, m_end;
    const uint16_t *w = g.w;
    if (g.tiles) {
        if ((int)blockIdx.y >= *g.n_tiles) return;
        const FhTile t = g.tiles[blockIdx.y];
        row0 = t.row0;
        m_end = t.row0 + t.rows;
        w += (int64_t)t.group * g.w_group;
    } else {
        row0 = (int)blockIdx.y * BM;
        m_end = g.m;
    }
    const int n0 = (int)blockIdx.x * BN, r = tid >> 2, c = (tid & 3) * 8;
    const int n = n0 + r < g.n ? n0 + r : g.n - 1;
    int m = row0 + r < m_end ? row0 + r : m_end - 1;
    if (g.gather) m = g.gather[m];
    const uint16_t *wp = w + (int64_t)n * g.kp + c;
    const float *xp = (const float *)g.x + (int64_t)m * g.kp + c;
    fh_f4 acc[2][2];
#pragma unroll
    for (int a = 0; a < 2; a++)
#pragma unroll
        for (int b = 0; b < 2; b++) acc[a][b] = fh_f4{0.f, 0.f, 0.f, 0.f};
    uint4 rw = *(const uint4 *)wp;
    float4 rx0 = *(const float4 *)xp, rx1 = *(const float4 *)(xp + 4);
    for (int k = 0; k < g.kp; k += 32) {
        float *d = sw_ + r * LD + c;
        *(float4 *)d = make_float4(fh_bf_lo(rw.x), fh_bf_hi(rw.x), fh_bf_lo(rw.y), fh_bf_hi(rw.y));
        *(float4 *)(d + 4) = make_float4(fh_bf_lo(rw.z), fh_bf_hi(rw.z), fh_bf_lo(rw.w), fh_bf_hi(rw.w));
        *(float4 *)(sx_ + r * LD + c) = rx0;
        *(float4 *)(sx_ + r * LD + c + 4) = rx1;
        __syncthreads();
        if (k + 32 < g.kp) {
            rw = *(const uint4 *)(wp + k + 32);
            rx0 = *(const float4 *)(xp + k + 32);
            rx1 = *(const float4 *)(xp + k + 36);
        }
        fh_f8 fw[2], fx[2];
#pragma unroll
        for (int a = 0; a < 2; a++) {
            fh_frag_load(fw[a], sw_ + (wn * 32 + a * 16 + li) * LD + gq * 8);
            fh_frag_load(fx[a], sx_ + (wm * 32 + a * 16 + li) * LD + gq * 8);
        }
#pragma unroll
        for (int a = 0; a < 2; a++)
#pragma unroll
            for (int b = 0; b < 2; b++)
                acc[a][b] = EPI == FH_GEMM_ACT_T ? fh_mma32(fx[b], fw[a], acc[a][b]) : fh_mma32(fw[a], fx[b], acc[a][b]);
        __syncthreads();
    }
#pragma unroll
    for (int b = 0; b < 2; b++) {
        const int mb = row0 + wm * 32 + b * 16;
        if (EPI == FH_GEMM_SWIGLU) {
            fh_f4 v;
#pragma unroll
            for (int e = 0; e < 4; e++) v[e] = fh_silu_f(acc[0][b][e]) * acc[1][b][e];
            gemm_store<FH_GEMM_ACT, float>(g.y, g.ldy, mb + li, (n0 + wn * 32) / 2 + gq * 4, v, m_end, g.n / 2);
        } else {
#pragma unroll
            for (int a = 0; a < 2; a++) {
                const int nb = n0 + wn * 32 + a * 16;
                if (EPI == FH_GEMM_ACT_T) gemm_store<EPI, float>(g.y, g.ldy, mb + gq * 4, nb + li, acc[a][b], m_end, g.n);
                else if (EPI == FH_GEMM_RELU2) gemm_store<FH_GEMM_ACT, float>(g.y, g.ldy, mb + li, nb + gq * 4, relu2(acc[a][b]), m_end, g.n);
                else gemm_store<EPI, float>(g.y, g.ldy, mb + li, nb + gq * 4, acc[a][b], m_end, g.n);
            }
        }
    }
}

fh_status fh_gemm(fh_device *dev, int dtype, int epi, const FhGemm &g) {
    FH_REQUIRE(g.w && g.x && g.y && g.n > 0 && g.kp > 0 && g.kp % 64 == 0, "bad product");
    FH_REQUIRE(g.tiles ? g.max_tiles > 0 && g.n_tiles : g.m > 0, "product without rows");
    FH_REQUIRE(epi != FH_GEMM_SWIGLU || g.n % 32 == 0, "gate and up rows come in groups of 16");
    FH_REQUIRE(!g.tiles || g.tile_rows == 64 || (g.tile_rows == 128 && dtype != FH_F32), "row tiles of %d", g.tile_rows);
    FH_REQUIRE(epi != FH_GEMM_ACT_T || !g.tiles, "a grouped product has no transposed form");
    hipStream_t s = dev->stream;
#define FH_GEMM_EPI(K_, GRID_)                                              \
    switch (epi) {                                                          \
    case FH_GEMM_F32: K_(FH_GEMM_F32)<<<GRID_, 256, 0, s>>>(g); break;      \
    case FH_GEMM_ACT: K_(FH_GEMM_ACT)<<<GRID_, 256, 0, s>>>(g); break;      \
    case FH_GEMM_ACT_T: K_(FH_GEMM_ACT_T)<<<GRID_, 256, 0, s>>>(g); break;  \
    case FH_GEMM_RELU2: K_(FH_GEMM_RELU2)<<<GRID_, 256, 0, s>>>(g); break;  \
    default: K_(FH_GEMM_SWIGLU)<<<GRID_, 256, 0, s>>>(g); break;            \
    }
    if (dtype == FH_F32) {
        const int ty = g.tiles ? g.max_tiles : (g.m + 63) / 64;
        FH_REQUIRE(ty <= 65535, "too many rows for one launch");
        const dim3 grid((unsigned)((g.n + 63) / 64), (unsigned)ty);
#define FH_K_(E_) k_gemm_f32<E_>
        FH_GEMM_EPI(FH_K_, grid)
#undef FH_K_
    } else {
        const int tn = (g.n + 127) / 128;
        // small row tiles where the large ones would leave compute units without work
        const bool big = g.tiles ? g.tile_rows == 128 : (int64_t)tn * ((g.m + 127) / 128) >= dev->compute_units;
        const int ty = g.tiles ? g.max_tiles : big ? (g.m + 127) / 128 : (g.m + 63) / 64;
        FH_REQUIRE(ty <= 65535, "too many rows for one launch");
        const dim3 grid((unsigned)tn, (unsigned)ty);
        if (big) {
#define FH_K_(E_) k_gemm_bf16<128, E_>
            FH_GEMM_EPI(FH_K_, grid)
#undef FH_K_
        } else {
#define FH_K_(E_) k_gemm_bf16<64, E_>
            FH_GEMM_EPI(FH_K_, grid)
#undef FH_K_
        }
    }
#undef FH_GEMM_EPI
    FH_HIP(hipGetLastError());
    return FH_OK;
}

// ------------------------------------------------------------------------------ rows -> activation rows
template <typename T>
__global__ __launch_bounds__(256) void k_rows_to_act(const float *__restrict__ x, int64_t ldx, int k, const float *__restrict__ w,
                                                     float eps, T *__restrict__ y, int kp) {
    __shared__ float red[4];
    const float *xr = x + (int64_t)blockIdx.x * ldx;
    T *yr = y + (int64_t)blockIdx.x * kp;
    float inv = 1.f;
    if (w) {
        float ss = 0.f;
        for (int i = threadIdx.x; i < k; i += 256) ss = fmaf(xr[i], xr[i], ss);
        ss = fh_wave_sum(ss);
        if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
        __syncthreads();
        inv = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)k + eps);
    }
    for (int i = threadIdx.x; i < kp; i += 256) {
        float v = i < k ? xr[i] : 0.f;
        if (w && i < k) v = v * inv * w[i];
        yr[i] = fh_to<T>(v);
    }
}

fh_status fh_rows_to_act(fh_device *dev, int dtype, const float *x, int64_t ldx, int rows, int k, const float *w, float eps,
                         void *y, int kp) {
    if (dtype == FH_F32)
        k_rows_to_act<float><<<dim3((unsigned)rows), 256, 0, dev->stream>>>(x, ldx, k, w, eps, (float *)y, kp);
    else
        k_rows_to_act<uint16_t><<<dim3((unsigned)rows), 256, 0, dev->stream>>>(x, ldx, k, w, eps, (uint16_t *)y, kp);
    FH_HIP(hipGetLastError());
    return FH_OK;
}

// ------------------------------------------------------------------------------ decode matvec
// One wavefront per ROWS weight rows; a lane takes eight consecutive weights (16 bytes) of every 512.  The input is
// normed once per workgroup into the LDS; f32 products and sums.
struct MvSegs { FhMvSeg s[3]; int tiles[3]; int n; };

template <int ROWS>
__global__ __launch_bounds__(256) void k_matvec_norm(const float *__restrict__ x, int k, int kp, const float *__restrict__ nw,
                                                     float eps, MvSegs segs, float *__restrict__ norm_out) {
    extern __shared__ __attribute__((aligned(16))) float xs[]; // [kp]
    __shared__ float red[4];
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    int tile = blockIdx.x, si = 0;
    while (si + 1 < segs.n && tile >= segs.tiles[si]) tile -= segs.tiles[si++];
    const FhMvSeg seg = segs.s[si];
    const int row0 = (tile * 4 + wave) * ROWS;
    const uint16_t *wr[ROWS];
#pragma unroll
    for (int r = 0; r < ROWS; r++) wr[r] = seg.w + (int64_t)(row0 + r < seg.n ? row0 + r : seg.n - 1) * kp + lane * 8;
    // the first weights are requested before the norm
    uint4 cur[ROWS];
    const bool in0 = lane * 8 < kp;
#pragma unroll
    for (int r = 0; r < ROWS; r++) cur[r] = in0 ? *(const uint4 *)wr[r] : uint4{0, 0, 0, 0};
    float ss = 0.f;
    if ((k & 3) == 0) {
#pragma unroll 4
        for (int i = tid * 4; i < kp; i += 1024) {
            const float4 v = i < k ? *(const float4 *)(x + i) : make_float4(0.f, 0.f, 0.f, 0.f);
            ss = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, ss))));
            *(float4 *)(xs + i) = v;
        }
    } else {
        for (int i = tid; i < kp; i += 256) {
            const float v = i < k ? x[i] : 0.f;
            ss = fmaf(v, v, ss);
            xs[i] = v;
        }
    }
    if (nw) {
        ss = fh_wave_sum(ss);
        if (lane == 0) red[wave] = ss;
        __syncthreads();
        const float inv = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)k + eps);
#pragma unroll 4
        for (int i = tid; i < k; i += 256) xs[i] = xs[i] * inv * nw[i];
    }
    __syncthreads();
    if (norm_out && blockIdx.x == 0)
        for (int i = tid; i < kp; i += 256) norm_out[i] = xs[i];
    float acc[ROWS];
#pragma unroll
    for (int r = 0; r < ROWS; r++) acc[r] = 0.f;
    for (int c = lane * 8; c < kp; c += 512) {
        uint4 nxt[ROWS];
        const bool more = c + 512 < kp;
#pragma unroll
        for (int r = 0; r < ROWS; r++) nxt[r] = more ? *(const uint4 *)(wr[r] + (c - lane * 8) + 512) : uint4{0, 0, 0, 0};
        const float4 a = *(const float4 *)(xs + c), b = *(const float4 *)(xs + c + 4);
#pragma unroll
        for (int r = 0; r < ROWS; r++) {
            acc[r] = fmaf(fh_bf_lo(cur[r].x), a.x, acc[r]);
            acc[r] = fmaf(fh_bf_hi(cur[r].x), a.y, acc[r]);
            acc[r] = fmaf(fh_bf_lo(cur[r].y), a.z, acc[r]);
            acc[r] = fmaf(fh_bf_hi(cur[r].y), a.w, acc[r]);
            acc[r] = fmaf(fh_bf_lo(cur[r].z), b.x, acc[r]);
            acc[r] = fmaf(fh_bf_hi(cur[r].z), b.y, acc[r]);
            acc[r] = fmaf(fh_bf_lo(cur[r].w), b.z, acc[r]);
            acc[r] = fmaf(fh_bf_hi(cur[r].w), b.w, acc[r]);
            cur[r] = nxt[r];
        }
    }
#pragma unroll
    for (int r = 0; r < ROWS; r++) acc[r] = fh_wave_sum(acc[r]);
    if (lane == 0)
#pragma unroll
        for (int r = 0; r < ROWS; r++)
            if (row0 + r < seg.n) seg.y[row0 + r] = acc[r];
}

fh_status fh_matvec_norm(fh_device *dev, const float *x, int k, const float *w, float eps, const FhMvSeg *segs, int n_segs,
                         float *norm_out) {
    FH_REQUIRE(n_segs >= 1 && n_segs <= 3, "1 to 3 matrices per matvec launch");
    const int kp = (int)fh_pad64(k);
    MvSegs ms{};
    int64_t total = 0;
    for (int i = 0; i < n_segs; i++) total += segs[i].n;
    const int rows = total >= (int64_t)dev->compute_units * 4 * 4 * 2 ? 4 : total >= (int64_t)dev->compute_units * 4 * 2 ? 2 : 1;
    int tiles = 0;
    ms.n = n_segs;
    for (int i = 0; i < n_segs; i++) {
        ms.s[i] = segs[i];
        ms.tiles[i] = (segs[i].n + 4 * rows - 1) / (4 * rows);
        tiles += ms.tiles[i];
    }
    const size_t lds = (size_t)kp * 4;
    FH_REQUIRE(lds <= 120 * 1024, "k = %d too long for the matvec", k);
    const void *fn = rows == 4 ? (const void *)k_matvec_norm<4> : rows == 2 ? (const void *)k_matvec_norm<2> : (const void *)k_matvec_norm<1>;
    if (lds > 48 * 1024) FH_TRY(fh_kernel_lds(dev, fn, lds));
    if (rows == 4) k_matvec_norm<4><<<dim3((unsigned)tiles), 256, lds, dev->stream>>>(x, k, kp, w, eps, ms, norm_out);
    else if (rows == 2) k_matvec_norm<2><<<dim3((unsigned)tiles), 256, lds, dev->stream>>>(x, k, kp, w, eps, ms, norm_out);
    else k_matvec_norm<1><<<dim3((unsigned)tiles), 256, lds, dev->stream>>>(x, k, kp, w, eps, ms, norm_out);
    FH_HIP(hipGetLastError());
    return FH_OK;
}

// ------------------------------------------------------------------------------ residual streams normed at a sublayer's end
__global__ void k_group_tiles(int groups, int s, int tile_rows, FhTile *tiles, int *n_tiles) {
    const int per = (s + tile_rows - 1) / tile_rows;
    for (int i = threadIdx.x; i < groups * per; i += blockDim.x) {
        const int g = i / per, r = i % per * tile_rows;
        tiles[i] = FhTile{g, g * s + r, s - r < tile_rows ? s - r : tile_rows, 0};
    }
    if (threadIdx.x == 0) *n_tiles = groups * per;
}

fh_status fh_group_tiles(fh_device *dev, int groups, int s, int tile_rows, FhTile *tiles, int *n_tiles) {
    k_group_tiles<<<1, 256, 0, dev->stream>>>(groups, s, tile_rows, tiles, n_tiles);
    FH_HIP(hipGetLastError());
    return FH_OK;
}

template <typename T>
__global__ __launch_bounds__(256) void k_add_normed(const float *__restrict__ x, const float *__restrict__ y, int k,
                                                    const float *__restrict__ w, float eps, float *__restrict__ x_out,
                                                    T *__restrict__ act, int kp) {
    constexpr int R = 16; // values of a thread that are requested at once; longer rows are read twice
    __shared__ float red[4];
    const int64_t row = (int64_t)blockIdx.x * k;
    float xv[R], yv[R], wv[R], ss = 0.f;
#pragma unroll
    for (int j = 0; j < R; j++) {
        const int i = threadIdx.x + 256 * j;
        const bool ok = i < k;
        yv[j] = ok ? y[row + i] : 0.f;
        xv[j] = ok ? x[row + i] : 0.f;
        wv[j] = ok ? w[i] : 0.f;
    }
#pragma unroll
    for (int j = 0; j < R; j++) ss = fmaf(yv[j], yv[j], ss);
    for (int i = threadIdx.x + 256 * R; i < k; i += 256) ss = fmaf(y[row + i], y[row + i], ss);
    ss = fh_wave_sum(ss);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    const float inv = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)k + eps);
    T *ar = act + (int64_t)blockIdx.x * kp;
#pragma unroll
    for (int j = 0; j < R; j++) {
        const int i = threadIdx.x + 256 * j;
        const float v = xv[j] + yv[j] * inv * wv[j];
        if (i < k) x_out[row + i] = v;
        if (act && i < kp) ar[i] = fh_to<T>(v); // zeros from k on
    }
    for (int i = threadIdx.x + 256 * R; i < kp; i += 256) {
        float v = 0.f;
        if (i < k) x_out[row + i] = v = x[row + i] + y[row + i] * inv * w[i];
        if (act) ar[i] = fh_to<T>(v);
    }
}

fh_status fh_add_normed(fh_device *dev, int dtype, const float *x, const float *y, int rows, int k, const float *w, float eps,
                        float *x_out, void *act, int kp) {
    const dim3 grid((unsigned)rows);
    if (dtype == FH_F32) k_add_normed<float><<<grid, 256, 0, dev->stream>>>(x, y, k, w, eps, x_out, (float *)act, kp);
    else k_add_normed<uint16_t><<<grid, 256, 0, dev->stream>>>(x, y, k, w, eps, x_out, (uint16_t *)act, kp);
    FH_HIP(hipGetLastError());
    return FH_OK;
}

template <typename T>
__global__ __launch_bounds__(256) void k_embed_at(const uint16_t *__restrict__ table, int n, const uint16_t *__restrict__ pos_table,
                                                  int positions, const uint32_t *__restrict__ ids, int pos,
                                                  const int *__restrict__ pos_dev, int k, float *__restrict__ x, T *__restrict__ act, int kp) {
    const int t = blockIdx.y, c = (int)blockIdx.x * 256 + threadIdx.x;
    if (c >= kp) return;
    const uint32_t id = ids[t];
    int p = (pos_dev ? *pos_dev : pos) + t;
    p = p < positions ? p : positions - 1; // the host refuses positions behind the table
    float v = 0.f;
    if (c < k) {
        v = fh_bf_f32(table[(int64_t)(id < (uint32_t)n ? id : 0) * kp + c]);
        if (pos_table) v += fh_bf_f32(pos_table[(int64_t)p * kp + c]);
        x[(int64_t)t * k + c] = v;
    }
    if (act) act[(int64_t)t * kp + c] = fh_to<T>(v);
}

fh_status fh_embed_at(fh_device *dev, int dtype, const fh_qmatrix *table, const fh_qmatrix *pos_table, const uint32_t *ids, int s,
                      int pos, const int *pos_dev, float *x, void *act, int kp) {
    FH_REQUIRE(table->type == FH_BF16 && table->recs == kp && (!pos_table || (pos_table->type == FH_BF16 && pos_table->recs == kp)),
               "embedding tables are bf16 rows of one stride");
    const dim3 grid((unsigned)((kp + 255) / 256), (unsigned)s);
    const uint16_t *tb = (const uint16_t *)table->data, *pt = pos_table ? (const uint16_t *)pos_table->data : nullptr;
    const int n = (int)table->n, np = pos_table ? (int)pos_table->n : 1 << 30, k = (int)table->k;
    if (dtype == FH_F32) k_embed_at<float><<<grid, 256, 0, dev->stream>>>(tb, n, pt, np, ids, pos, pos_dev, k, x, (float *)act, kp);
    else k_embed_at<uint16_t><<<grid, 256, 0, dev->stream>>>(tb, n, pt, np, ids, pos, pos_dev, k, x, (uint16_t *)act, kp);
    FH_HIP(hipGetLastError());
    return FH_OK;
}

template <typename T>
__global__ __launch_bounds__(256) void k_token_shift(FhShift m, const float *__restrict__ x, int k, int pos,
                                                     const float *__restrict__ state, int kp) {
    const int t = blockIdx.y, c = (int)blockIdx.x * 256 + threadIdx.x;
    if (c >= kp) return;
    float v = 0.f, d = 0.f;
    if (c < k) {
        v = x[(int64_t)t * k + c];
        d = (t > 0 ? x[(int64_t)(t - 1) * k + c] : pos > 0 ? state[((pos - 1) & 1) * k + c] : 0.f) - v;
    }
#pragma unroll
    for (int n = 0; n < FH_SHIFT_MAX; n++) {
        if (n >= m.n) break;
        const float y = c < k ? fmaf(d, m.mu[n][c], v) : 0.f;
        const int64_t o = (int64_t)t * kp + c;
        if (m.f32[n]) ((float *)m.y[n])[o] = y;
        else ((T *)m.y[n])[o] = fh_to<T>(y);
    }
}

fh_status fh_token_shift(fh_device *dev, int dtype, const FhShift &m, const float *x, int s, int k, int pos, float *state, int kp) {
    const dim3 grid((unsigned)((kp + 255) / 256), (unsigned)s);
    if (dtype == FH_F32) k_token_shift<float><<<grid, 256, 0, dev->stream>>>(m, x, k, pos, state, kp);
    else k_token_shift<uint16_t><<<grid, 256, 0, dev->stream>>>(m, x, k, pos, state, kp);
    FH_HIP(hipGetLastError());
    // after every reader of the old rows
    return fh_copy(dev, state + (int64_t)((pos + s - 1) & 1) * k, x + (int64_t)(s - 1) * k, (size_t)k * 4);
}

// A workgroup takes 16 rows of x and 16 of W; its four wavefronts share out k.  True f32 products on the widened weights.
__global__ __launch_bounds__(256) void k_low_rank_tanh(const float *__restrict__ x, int kp, int rows, const uint16_t *__restrict__ w, int n,
                                                       float *__restrict__ y, int ldy) {
    __shared__ float red[4][256];
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, li = lane & 15, g = lane >> 4, m0 = (int)blockIdx.x * 16, n0 = (int)blockIdx.y * 16;
    const float *xp = x + (int64_t)(m0 + li < rows ? m0 + li : rows - 1) * kp + 8 * g;
    const uint16_t *wp = w + (int64_t)(n0 + li < n ? n0 + li : n - 1) * kp + 8 * g;
    fh_f4 acc = fh_f4{0.f, 0.f, 0.f, 0.f};
    for (int k = 32 * wave; k < kp; k += 128) {
        const uint4 u = *(const uint4 *)(wp + k);
        const fh_f8 fw = {{fh_bf_lo(u.x), fh_bf_hi(u.x), fh_bf_lo(u.y), fh_bf_hi(u.y), fh_bf_lo(u.z), fh_bf_hi(u.z), fh_bf_lo(u.w), fh_bf_hi(u.w)}};
        fh_f8 fx;
        fh_frag_load(fx, xp + k);
        acc = fh_mma32(fw, fx, acc); // a lane: W rows 4 g .. + 3 of x row li
    }
#pragma unroll
    for (int e = 0; e < 4; e++) red[wave][lane * 4 + e] = acc[e];
    __syncthreads();
    const int r = m0 + (tid >> 2) % 16, c = n0 + 4 * (tid >> 6) + (tid & 3); // lane tid / 4, element tid % 4
    const float v = (red[0][tid] + red[1][tid]) + (red[2][tid] + red[3][tid]);
    if (r < rows && c < ldy) y[(int64_t)r * ldy + c] = c < n ? tanhf(v) : 0.f;
}

fh_status fh_low_rank_tanh(fh_device *dev, const float *x, int kp, int rows, const uint16_t *w, int n, float *y, int ldy) {
    FH_REQUIRE(n > 0 && ldy >= n && kp % 64 == 0, "bad low-rank product");
    k_low_rank_tanh<<<dim3((unsigned)((rows + 15) / 16), (unsigned)((ldy + 15) / 16)), 256, 0, dev->stream>>>(x, kp, rows, w, n, y, ldy);
    FH_HIP(hipGetLastError());
    return FH_OK;
}

// A workgroup of eight wavefronts works its input out once, into the LDS; one wavefront per ROWS weight rows, a lane takes
// eight consecutive weights (16 bytes) of every 512.  The first AHEAD pieces of 512 are requested before the input, later ones
// while earlier ones are multiplied.
struct MvMixes { FhMvMix s[FH_MV_MAX]; int tiles[FH_MV_MAX]; int n; };

__device__ __forceinline__ float mv_sum8(const float *red) {
    return ((red[0] + red[1]) + (red[2] + red[3])) + ((red[4] + red[5]) + (red[6] + red[7]));
}

// x' into the LDS, mixed with the token before it where the matrix wants that.
__device__ __forceinline__ void mv_input(const FhMvAdd &in, const float *mu, int k, int kp, float *xs, float *red) {
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const int pos = in.state ? *in.pos_dev : 0;
    const float *before = in.state + ((pos - 1) & 1) * k;
    float *here = in.state + (pos & 1) * k;
    const bool one = blockIdx.x == 0, shift = mu && pos > 0;
    if (!(k & 3) && k <= 4096) { // everything is requested at once
        float4 x[2], y[2], w[2], m[2], b[2];
        const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < 2; j++) {
            const int i = (tid + 512 * j) * 4;
            const bool ok = i < k;
            x[j] = ok ? *(const float4 *)(in.x + i) : zero;
            y[j] = ok && in.y ? *(const float4 *)(in.y + i) : zero;
            w[j] = ok && in.y ? *(const float4 *)(in.w + i) : zero;
            m[j] = ok && mu ? *(const float4 *)(mu + i) : zero;
            b[j] = ok && shift ? *(const float4 *)(before + i) : zero;
        }
        float inv = 0.f;
        if (in.y) {
#pragma unroll
            for (int j = 0; j < 2; j++) ss = fmaf(y[j].x, y[j].x, fmaf(y[j].y, y[j].y, fmaf(y[j].z, y[j].z, fmaf(y[j].w, y[j].w, ss))));
            ss = fh_wave_sum(ss);
            if (lane == 0) red[wave] = ss;
            __syncthreads();
            inv = 1.0f / sqrtf(mv_sum8(red) / (float)k + in.eps);
        }
#pragma unroll
        for (int j = 0; j < 2; j++) {
            const int i = (tid + 512 * j) * 4;
            if (i >= kp) break;
            float4 v = x[j];
            if (in.y) v = make_float4(v.x + y[j].x * inv * w[j].x, v.y + y[j].y * inv * w[j].y, v.z + y[j].z * inv * w[j].z, v.w + y[j].w * inv * w[j].w);
            if (one && i < k) {
                if (in.x_out) *(float4 *)(in.x_out + i) = v;
                if (in.state) *(float4 *)(here + i) = v;
            }
            if (mu)
                v = make_float4(fmaf(b[j].x - v.x, m[j].x, v.x), fmaf(b[j].y - v.y, m[j].y, v.y), fmaf(b[j].z - v.z, m[j].z, v.z),
                                fmaf(b[j].w - v.w, m[j].w, v.w));
            *(float4 *)(xs + i) = v;
        }
        return;
    }
    float inv = 0.f;
    if (in.y) {
        float ss = 0.f;
#pragma unroll 4
        for (int i = tid; i < k; i += 512) ss = fmaf(in.y[i], in.y[i], ss);
        ss = fh_wave_sum(ss);
        if (lane == 0) red[wave] = ss;
        __syncthreads();
        inv = 1.0f / sqrtf(mv_sum8(red) / (float)k + in.eps);
    } else if (!(k & 3) && !in.x_out && !in.state && !mu) { // a plain copy
#pragma unroll 4
        for (int i = tid * 4; i < kp; i += 2048) *(float4 *)(xs + i) = i < k ? *(const float4 *)(in.x + i) : make_float4(0.f, 0.f, 0.f, 0.f);
        return;
    }
    for (int i = tid; i < kp; i += 512) {
        float v = 0.f;
        if (i < k) {
            v = in.x[i];
            if (in.y) v += in.y[i] * inv * in.w[i];
            if (one) {
                if (in.x_out) in.x_out[i] = v;
                if (in.state) here[i] = v;
            }
            if (mu) v = fmaf((shift ? before[i] : 0.f) - v, mu[i], v);
        }
        xs[i] = v;
    }
}

// Normed group by group and gated.
__device__ __forceinline__ void mv_gated(const FhMvAdd &in, int k, int kp, float *xs, float *ginv) {
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, gl = k / in.groups;
#pragma unroll 4
    for (int i = tid; i < kp; i += 512) xs[i] = i < k ? in.x[i] : 0.f;
    __syncthreads();
    for (int g = wave; g < in.groups; g += 8) {
        float ss = 0.f;
        for (int i = lane; i < gl; i += 64) ss = fmaf(xs[g * gl + i], xs[g * gl + i], ss);
        ss = fh_wave_sum(ss);
        if (lane == 0) ginv[g] = 1.0f / sqrtf(ss / (float)gl + in.eps) * in.scale;
    }
    __syncthreads();
#pragma unroll 4
    for (int i = tid; i < k; i += 512) {
        float v = xs[i] * ginv[i / gl];
        if (in.w) v *= in.w[in.w_len == k ? i : i % in.w_len];
        xs[i] = v * fh_silu_f(in.gate[i]);
    }
}

template <int ROWS, bool GATED>
__global__ __launch_bounds__(512) void k_matvec_mix(FhMvAdd in, int k, int kp, MvMixes segs) {
    constexpr int AHEAD = ROWS == 4 ? 3 : 8 / ROWS;
    extern __shared__ __attribute__((aligned(16))) float xs[]; // [kp | groups]
    __shared__ float red[8];
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    int tile = blockIdx.x, si = 0;
    while (si + 1 < segs.n && tile >= segs.tiles[si]) tile -= segs.tiles[si++];
    const FhMvMix seg = segs.s[si];
    const int row0 = (tile * 8 + wave) * ROWS, pieces = (kp + 511) / 512;
    const uint16_t *wr[ROWS];
#pragma unroll
    for (int r = 0; r < ROWS; r++) wr[r] = seg.w + (int64_t)(row0 + r < seg.n ? row0 + r : seg.n - 1) * kp + lane * 8;
    uint4 u[AHEAD][ROWS];
    auto fetch = [&](int i, uint4 *v) {
        const bool ok = i * 512 + lane * 8 < kp;
#pragma unroll
        for (int r = 0; r < ROWS; r++) v[r] = ok ? *(const uint4 *)(wr[r] + i * 512) : uint4{0, 0, 0, 0};
    };
#pragma unroll
    for (int i = 0; i < AHEAD; i++) fetch(i, u[i]);
    if (GATED) mv_gated(in, k, kp, xs, xs + kp);
    else mv_input(in, seg.mu, k, kp, xs, red);
    __syncthreads();
    float acc[ROWS];
#pragma unroll
    for (int r = 0; r < ROWS; r++) acc[r] = 0.f;
    for (int p = 0; p < pieces; p += AHEAD) {
#pragma unroll
        for (int i = 0; i < AHEAD; i++) {
            uint4 cur[ROWS];
#pragma unroll
            for (int r = 0; r < ROWS; r++) cur[r] = u[i][r];
            fetch(p + i + AHEAD, u[i]);
            const int c = (p + i) * 512 + lane * 8;
            if (c >= kp) continue;
            const float4 a = *(const float4 *)(xs + c), b = *(const float4 *)(xs + c + 4);
#pragma unroll
            for (int r = 0; r < ROWS; r++) {
                acc[r] = fmaf(fh_bf_lo(cur[r].x), a.x, acc[r]);
                acc[r] = fmaf(fh_bf_hi(cur[r].x), a.y, acc[r]);
                acc[r] = fmaf(fh_bf_lo(cur[r].y), a.z, acc[r]);
                acc[r] = fmaf(fh_bf_hi(cur[r].y), a.w, acc[r]);
                acc[r] = fmaf(fh_bf_lo(cur[r].z), b.x, acc[r]);
                acc[r] = fmaf(fh_bf_hi(cur[r].z), b.y, acc[r]);
                acc[r] = fmaf(fh_bf_lo(cur[r].w), b.z, acc[r]);
                acc[r] = fmaf(fh_bf_hi(cur[r].w), b.w, acc[r]);
            }
        }
    }
#pragma unroll
    for (int r = 0; r < ROWS; r++) acc[r] = fh_wave_sum(acc[r]);
    if (lane == 0)
#pragma unroll
        for (int r = 0; r < ROWS; r++)
            if (row0 + r < seg.n) {
                float v = acc[r];
                if (seg.act == FH_MV_ACT_RELU2) v = fmaxf(v, 0.f) * fmaxf(v, 0.f);
                else if (seg.act == FH_MV_ACT_TANH) v = tanhf(v);
                seg.y[row0 + r] = v;
            }
}

template <int ROWS, bool GATED>
static fh_status matvec_mix_go(fh_device *dev, const FhMvAdd &in, int k, int kp, const MvMixes &ms, int tiles) {
    const size_t lds = (size_t)(kp + (GATED ? in.groups : 0)) * 4;
    FH_REQUIRE(lds <= 150 * 1024, "k = %d too long for the matvec", k);
    if (lds > 48 * 1024) FH_TRY(fh_kernel_lds(dev, (const void *)k_matvec_mix<ROWS, GATED>, lds));
    k_matvec_mix<ROWS, GATED><<<dim3((unsigned)tiles), 512, lds, dev->stream>>>(in, k, kp, ms);
    FH_HIP(hipGetLastError());
    return FH_OK;
}

fh_status fh_matvec_mix(fh_device *dev, const FhMvAdd &in, int k, const FhMvMix *segs, int n_segs) {
    FH_REQUIRE(n_segs >= 1 && n_segs <= FH_MV_MAX, "1 to %d matrices per launch", FH_MV_MAX);
    FH_REQUIRE(in.x && in.x != in.x_out && (!in.y || in.w) && (!in.state || in.pos_dev), "bad input of a decode product");
    FH_REQUIRE(!in.gate || (!in.y && !in.state && in.groups > 0 && k % in.groups == 0), "bad gated input of a decode product");
    const int kp = (int)fh_pad64(k);
    MvMixes ms{};
    int64_t total = 0;
    for (int i = 0; i < n_segs; i++) total += segs[i].n;
    const int rows = total >= (int64_t)dev->compute_units * 8 * 4 ? 4 : total >= (int64_t)dev->compute_units * 8 * 2 ? 2 : 1;
    int tiles = 0;
    ms.n = n_segs;
    for (int i = 0; i < n_segs; i++) {
        ms.s[i] = segs[i];
        ms.tiles[i] = (segs[i].n + 8 * rows - 1) / (8 * rows);
        tiles += ms.tiles[i];
    }
    if (in.gate)
        return rows == 4 ? matvec_mix_go<4, true>(dev, in, k, kp, ms, tiles) : rows == 2 ? matvec_mix_go<2, true>(dev, in, k, kp, ms, tiles)
                                                                                        : matvec_mix_go<1, true>(dev, in, k, kp, ms, tiles);
    return rows == 4 ? matvec_mix_go<4, false>(dev, in, k, kp, ms, tiles) : rows == 2 ? matvec_mix_go<2, false>(dev, in, k, kp, ms, tiles)
                                                                                     : matvec_mix_go<1, false>(dev, in, k, kp, ms, tiles);
}

// ------------------------------------------------------------------------------ fh_qmatmul on bf16 rows
__global__ __launch_bounds__(256) void k_pad_bf16_rows(const uint16_t *__restrict__ x, int k, uint16_t *__restrict__ y, int kp) {
    for (int i = threadIdx.x; i < kp; i += 256) y[(int64_t)blockIdx.x * kp + i] = i < k ? x[(int64_t)blockIdx.x * k + i] : 0;
}

// f32 activations are multiplied in true f32, bf16 ones on the bf16 matrix cores.
fh_status fh_launch_bf16_matmul(const fh_qmatrix *q, const void *x, int x_is_bf16, int m, float *y) {
    fh_device *dev = q->dev;
    const int k = (int)q->k, kp = (int)q->recs;
    if (m == 1 && !x_is_bf16 && (size_t)kp * 4 <= 120 * 1024) {
        const FhMvSeg s{(const uint16_t *)q->data, y, (int)q->n};
        return fh_matvec_norm(dev, (const float *)x, k, nullptr, 0.f, &s, 1, nullptr);
    }
    const int dt = x_is_bf16 ? FH_BF16_ACT : FH_F32;
    FH_TRY(fh_dev_scratch(dev, &dev->act_buf, &dev->act_cap, (size_t)m * kp * fh_act_size(dt)));
    if (x_is_bf16) {
        k_pad_bf16_rows<<<dim3((unsigned)m), 256, 0, dev->stream>>>((const uint16_t *)x, k, (uint16_t *)dev->act_buf, kp);
        FH_HIP(hipGetLastError());
    } else FH_TRY(fh_rows_to_act(dev, FH_F32, (const float *)x, k, m, k, nullptr, 0.f, dev->act_buf, kp));
    FhGemm g;
    g.w = (const uint16_t *)q->data, g.x = dev->act_buf, g.y = y, g.ldy = q->n, g.n = (int)q->n, g.kp = kp, g.m = m;
    return fh_gemm(dev, dt, FH_GEMM_F32, g);
}
