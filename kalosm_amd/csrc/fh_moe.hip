// Prefill of the mixture-of-experts feed-forward (fh_moe.h): routing, assignments sorted by expert, grouped products,
// and the weighted sum into the residual stream.
#include "fh_moe.h"

__global__ __launch_bounds__(256) void k_moe_route(FhMoe m, const float *__restrict__ proj, int64_t ldp, int s,
                                                   int *__restrict__ ids, float *__restrict__ wts) {
    const int t = (int)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (t >= s) return;
    fh_moe_route(proj + (int64_t)t * ldp + m.col_z, m.experts, m.scale, m.top, [&](int n, int e, float w) {
        if ((threadIdx.x & 63) == 0) ids[(int64_t)t * m.top + n] = e, wts[(int64_t)t * m.top + n] = w;
    });
}

// Counting sort of the assignments by expert, one workgroup; the order inside an expert is arbitrary (a row's result
// does not depend on its place).  Then the table of row tiles, none of which crosses an expert.
__global__ __launch_bounds__(1024) void k_moe_sort(FhMoe m, const int *__restrict__ ids, int s, int tile_rows,
                                                   int *__restrict__ src, int *__restrict__ inv, FhTile *__restrict__ tiles,
                                                   int *__restrict__ n_tiles) {
    __shared__ int count[FH_MOE_MAX_EXPERTS], start[FH_MOE_MAX_EXPERTS], tstart[FH_MOE_MAX_EXPERTS];
    const int tid = threadIdx.x, n = s * m.top;
    for (int e = tid; e < m.experts; e += 1024) count[e] = 0;
    __syncthreads();
    for (int i = tid; i < n; i += 1024) atomicAdd(&count[ids[i]], 1);
    __syncthreads();
    if (tid == 0) {
        int at = 0, tt = 0;
        for (int e = 0; e < m.experts; e++) {
            start[e] = at;
            tstart[e] = tt;
            at += count[e];
            tt += (count[e] + tile_rows - 1) / tile_rows;
        }
        *n_tiles = tt;
    }
    __syncthreads();
    for (int e = tid; e < m.experts; e += 1024)
        for (int i = 0, o = 0; o < count[e]; i++, o += tile_rows)
            tiles[tstart[e] + i] = FhTile{e, start[e] + o, count[e] - o < tile_rows ? count[e] - o : tile_rows, 0};
    __syncthreads();
    for (int e = tid; e < m.experts; e += 1024) count[e] = 0;
    __syncthreads();
    for (int i = tid; i < n; i += 1024) {
        const int e = ids[i], p = start[e] + atomicAdd(&count[e], 1);
        src[p] = i / m.top;
        inv[i] = p;
    }
}

// x += mix + the token's weighted expert rows + its row of the always-on expert
__global__ __launch_bounds__(256) void k_moe_combine(FhMoe m, const float *__restrict__ mix, const float *__restrict__ y,
                                                     const float *__restrict__ sy, const int *__restrict__ inv,
                                                     const float *__restrict__ wts, int width, float *__restrict__ x) {
    const int t = blockIdx.y, c = (int)blockIdx.x * 256 + threadIdx.x;
    if (c >= width) return;
    const int64_t o = (int64_t)t * width + c;
    float f = 0.f;
    for (int j = 0; j < m.top; j++) {
        const int64_t a = (int64_t)t * m.top + j;
        f = fmaf(wts[a], y[(int64_t)inv[a] * width + c], f);
    }
    if (sy) f += sy[o];
    x[o] += mix[o] + f;
}

fh_status fh_moe_prefill(fh_device *dev, int dtype, const FhMoe &m, const void *h, int kp, const float *proj, int64_t ldp,
                         int s, int width, const FhMoeWork &w, const float *mix, float *x) {
    hipStream_t str = dev->stream;
    if (m.experts) {
        const int tr = fh_moe_tile_rows(m, dtype, s);
        k_moe_route<<<dim3((unsigned)((s + 3) / 4)), 256, 0, str>>>(m, proj, ldp, s, w.ids, w.wts);
        k_moe_sort<<<dim3(1), 1024, 0, str>>>(m, w.ids, s, tr, w.src, w.inv, w.tiles, w.n_tiles);
        FH_HIP(hipGetLastError());
        FhGemm g;
        g.tiles = w.tiles;
        g.n_tiles = w.n_tiles;
        g.max_tiles = fh_moe_max_tiles(m, s, tr);
        g.tile_rows = tr;
        g.w = m.gate_up, g.w_group = m.gu_stride, g.n = 2 * m.ffp, g.kp = kp;
        g.x = h, g.gather = w.src, g.y = w.act, g.ldy = m.ffp;
        FH_TRY(fh_gemm(dev, dtype, FH_GEMM_SWIGLU, g));
        g.w = m.down, g.w_group = m.down_stride, g.n = width, g.kp = m.ffp;
        g.x = w.act, g.gather = nullptr, g.y = w.y, g.ldy = width;
        FH_TRY(fh_gemm(dev, dtype, FH_GEMM_F32, g));
    }
    if (m.sff) {
        FhGemm g;
        g.m = s;
        g.w = m.s_gate_up, g.n = 2 * m.sffp, g.kp = kp, g.x = h, g.y = w.s_act, g.ldy = m.sffp;
        FH_TRY(fh_gemm(dev, dtype, FH_GEMM_SWIGLU, g));
        g.w = m.s_down, g.n = width, g.kp = m.sffp, g.x = w.s_act, g.y = w.s_y, g.ldy = width;
        FH_TRY(fh_gemm(dev, dtype, FH_GEMM_F32, g));
    }
    FhMoe mm = m;
    if (!m.experts) mm.top = 0;
    k_moe_combine<<<dim3((unsigned)((width + 255) / 256), (unsigned)s), 256, 0, str>>>(mm, mix, w.y, m.sff ? w.s_y : nullptr,
                                                                                      w.inv, w.wts, width, x);
    FH_HIP(hipGetLastError());
    return FH_OK;
}
