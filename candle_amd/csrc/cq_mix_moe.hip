// Mixture of experts with bfloat16 weights: choice of experts from router logits, the plan of a grouped product over many rows, and the single-token step
// that reads the chosen experts (and a shared one) straight from their stacked weights.
#include "cq_dense.h"
#include "cq_mix.h"

namespace {

constexpr int MAX_EXPERTS = CQ_MOE_MAX_EXPERTS, MAX_TOP = CQ_MOE_MAX_TOP;

// The `top` largest of n logits, largest first (the lower index of equals): lane j < top of the wave leaves with the id and the softmax weight, over the
// chosen ones only, of choice j.
template <int NV>
__device__ __forceinline__ void choose(const float *__restrict__ z, int n, int top, int lane, int &id, float &w) {
    float v[NV];
#pragma unroll
    for (int i = 0; i < NV; i++) v[i] = lane + 64 * i < n ? z[lane + 64 * i] : -INFINITY;
    float mine = -INFINITY, first = 0.0f;
    id = 0;
    for (int j = 0; j < top; j++) {
        float b = v[0];
#pragma unroll
        for (int i = 1; i < NV; i++) b = fmaxf(b, v[i]);
        const float m = wave_max(b);
        int at = 0x7fffffff;
#pragma unroll
        for (int i = NV - 1; i >= 0; i--) at = v[i] == m && lane + 64 * i < n ? lane + 64 * i : at;
        at = wave_min_int(at);
        at = at < n ? at : 0;                              // only with logits that are no numbers
#pragma unroll
        for (int i = 0; i < NV; i++) v[i] = lane + 64 * i == at ? -INFINITY : v[i];
        if (j == 0) first = m;
        if (lane == j) {
            mine = m;
            id = at;
        }
    }
    const float e = lane < top ? expf(mine - first) : 0.0f;
    w = e / wave_sum(e);
}
__device__ __forceinline__ void choose_any(const float *__restrict__ z, int n, int top, int lane, int &id, float &w) {
    if (n <= 64) choose<1>(z, n, top, lane, id, w);
    else if (n <= 256) choose<4>(z, n, top, lane, id, w);
    else choose<16>(z, n, top, lane, id, w);
}

// one wave per row
__global__ __launch_bounds__(256) void moe_select_kernel(const float *__restrict__ logits, int64_t ld, int64_t rows, int experts, int top, int shared,
                                                         int32_t *__restrict__ ids, float *__restrict__ weights, float *__restrict__ shared_weights) {
    const int lane = threadIdx.x & 63;
    const int64_t r = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (r >= rows) return;
    int id;
    float w;
    choose_any(logits + r * ld, experts, top, lane, id, w);
    if (lane < top) {
        ids[r * top + lane] = id;
        weights[r * top + lane] = w;
    }
    if (shared && lane == 0) shared_weights[r] = mix_sigmoid(logits[r * ld + experts]);
}

// One workgroup: pairs (row, choice) gathered by expert, cut into tiles of at most tile_rows.
__global__ __launch_bounds__(1024) void moe_plan_kernel(const int32_t *__restrict__ ids, const float *__restrict__ weights, int pairs, int experts, int top, int tile_rows,
                                                        int32_t *__restrict__ src_rows, int32_t *__restrict__ dst_rows, float *__restrict__ scale,
                                                        cq_dense_tile *__restrict__ tiles, int32_t *__restrict__ n_tiles) {
    __shared__ int count[MAX_EXPERTS], start[MAX_EXPERTS], tile0[MAX_EXPERTS], rows_in[16], tiles_in[16];
    const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
    if (tid < MAX_EXPERTS) count[tid] = 0;
    __syncthreads();
    // the first PER of a thread's ids stay in registers
    constexpr int PER = 16;
    int id[PER];
#pragma unroll
    for (int j = 0; j < PER; j++) id[j] = tid + 1024 * j < pairs ? ids[tid + 1024 * j] : -1;
#pragma unroll
    for (int j = 0; j < PER; j++)
        if (id[j] >= 0) atomicAdd(&count[id[j]], 1);
    for (int i = tid + 1024 * PER; i < pairs; i += 1024) atomicAdd(&count[ids[i]], 1);
    __syncthreads();
    // exclusive sums of rows and tiles over the experts: within the wave, then over the waves
    const int n = tid < experts ? count[tid] : 0, nt = (n + tile_rows - 1) / tile_rows;
    int a = n, b = nt;
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) {
        const int x = __shfl_up(a, d, 64), y = __shfl_up(b, d, 64);
        if (lane >= d) {
            a += x;
            b += y;
        }
    }
    if (lane == 63) {
        rows_in[wv] = a;
        tiles_in[wv] = b;
    }
    __syncthreads();
    int ra = 0, rb = 0;
    for (int i = 0; i < wv; i++) {
        ra += rows_in[i];
        rb += tiles_in[i];
    }
    a += ra - n;
    b += rb - nt;
    if (tid < experts) {
        start[tid] = a;
        tile0[tid] = b;
        for (int t = 0; t < nt; t++) {
            cq_dense_tile x;
            x.group = tid;
            x.first = a + t * tile_rows;
            x.rows = min(tile_rows, n - t * tile_rows);
            x.reserved = 0;
            tiles[b + t] = x;
        }
        if (tid == experts - 1) n_tiles[0] = b + nt;
    }
    __syncthreads();
    auto place = [&](int i, int e, float w) {
        const int at = atomicAdd(&start[e], 1);
        src_rows[at] = i / top;
        dst_rows[at] = i;
        scale[at] = w;
    };
    float w[PER];
#pragma unroll
    for (int j = 0; j < PER; j++) w[j] = id[j] >= 0 ? weights[tid + 1024 * j] : 0.0f;
#pragma unroll
    for (int j = 0; j < PER; j++)
        if (id[j] >= 0) place(tid + 1024 * j, id[j], w[j]);
    for (int i = tid + 1024 * PER; i < pairs; i += 1024) place(i, ids[i], weights[i]);
}

// x[r] += sum over the choices of y[r * top + j], in order
__global__ __launch_bounds__(256) void moe_add_kernel(const float *__restrict__ y, int64_t ldy, int top, float *__restrict__ x, int64_t ldx, int dim) {
    const int64_t r = blockIdx.x;
    const float *yr = y + r * top * ldy;
    float *xr = x + r * ldx;
    for (int i = threadIdx.x + 256 * blockIdx.y; 4 * i < dim; i += 256 * gridDim.y) {
        f32x4 a = *reinterpret_cast<const f32x4 *>(xr + 4 * i);
#pragma unroll 8
        for (int j = 0; j < top; j++) a += *reinterpret_cast<const f32x4 *>(yr + j * ldy + 4 * i);
        if (4 * i + 4 <= dim) *reinterpret_cast<f32x4 *>(xr + 4 * i) = a;
        else
#pragma unroll
            for (int e = 0; e < 4; e++)
                if (4 * i + e < dim) xr[4 * i + e] = a[e];
    }
}

// ---- one token ---------------------------------------------------------------------------------------------------------------------------------
// The choice, then weight * silu(gate) * up of every chosen expert and of the shared one: a wave takes (gate, up) pairs of rows, one block of loads ahead.  The
// input row sits in LDS, normalized.  Every workgroup chooses for itself; the first one leaves the ids for the second launch.
constexpr int UP_U = 4, UP_BLOCK = 512 * UP_U;
template <int NORM>
__global__ __launch_bounds__(512) void moe_up_step_kernel(cq_moe g, const float *__restrict__ x, const float *__restrict__ vec, float eps, int dim,
                                                          const float *__restrict__ logits, float *__restrict__ act, int32_t *__restrict__ ids_out) {
    extern __shared__ __attribute__((aligned(16))) float xs[];             // kp rounded up to UP_BLOCK
    __shared__ float red[8], cw[MAX_TOP + 1];
    __shared__ int32_t cid[MAX_TOP];
    const int tid = threadIdx.x, lane = tid & 63, wv = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int kb_n = (g.kp + UP_BLOCK - 1) / UP_BLOCK, n4 = kb_n * UP_BLOCK / 4;
    float s = 0.0f;
    for (int i = tid; i < n4; i += 512) {
        f32x4 v = *reinterpret_cast<const f32x4 *>(x + min(4 * i, g.kp - 4));
#pragma unroll
        for (int e = 0; e < 4; e++) {
            v[e] = 4 * i + e < dim ? v[e] : 0.0f;
            s += NORM == CQ_DENSE_LAYER_NORM ? v[e] : v[e] * v[e];
        }
        reinterpret_cast<f32x4 *>(xs)[i] = v;
    }
    if (wv == 0) {
        int id;
        float w;
        choose_any(logits, g.experts, g.top, lane, id, w);
        if (lane < g.top) {
            cid[lane] = id;
            cw[lane] = w;
            if (blockIdx.x == 0) ids_out[lane] = id;
        }
        if (lane == 0 && g.shared_ff) cw[g.top] = mix_sigmoid(logits[g.experts]);
    }
    if (NORM == CQ_DENSE_LAYER_NORM) {
        layer_norm_lds_512(xs, dim, s, vec, eps, red);
    } else {
        const float m = sqrtf(block_sum_512(s, red) / (float)dim + eps);
        for (int i = tid; i < dim; i += 512) xs[i] = xs[i] / m * vec[i];
    }
    __syncthreads();

    const int total = g.top * g.ff + g.shared_ff, step = gridDim.x * 8;
    int u = blockIdx.x * 8 + wv;
    auto row_of = [&](int p) -> const uint16_t * {
        if (p < g.top * g.ff) {
            const int slot = p / g.ff;
            return (const uint16_t *)g.up_dev + cid[slot] * g.up_stride + (int64_t)2 * (p - slot * g.ff) * g.kp;
        }
        return (const uint16_t *)g.shared_up_dev + (int64_t)2 * (p - g.top * g.ff) * g.kp;
    };
    u32x4 cur[2][UP_U], nxt[2][UP_U];
    auto load = [&](const uint16_t *p, int kb, u32x4 (&d)[2][UP_U]) {
#pragma unroll
        for (int t = 0; t < 2; t++)
#pragma unroll
            for (int i = 0; i < UP_U; i++)
                d[t][i] = __builtin_nontemporal_load(reinterpret_cast<const u32x4 *>(p + (int64_t)t * g.kp + min(kb * UP_BLOCK + i * 512 + lane * 8, g.kp - 8)));
    };
    if (u < total) load(row_of(u), 0, cur);
    for (; u < total; u += step) {
        float acc[2][2] = {};
        for (int kb = 0; kb < kb_n; kb++) {
            const bool last = kb + 1 == kb_n;
            const int next = last ? u + step : u;
            if (next < total) load(row_of(next), last ? 0 : kb + 1, nxt);
#pragma unroll
            for (int i = 0; i < UP_U; i++) {
                const f32x4 *xv = reinterpret_cast<const f32x4 *>(xs + kb * UP_BLOCK + i * 512 + lane * 8);
                const f32x4 a = xv[0], b = xv[1];
                dot8(cur[0][i], a, b, acc[0]);
                dot8(cur[1][i], a, b, acc[1]);
            }
#pragma unroll
            for (int t = 0; t < 2; t++)
#pragma unroll
                for (int i = 0; i < UP_U; i++) cur[t][i] = nxt[t][i];
        }
        const float gate = wave_sum(acc[0][0] + acc[0][1]), upv = wave_sum(acc[1][0] + acc[1][1]);
        if (lane == 0) {
            const int slot = u < g.top * g.ff ? u / g.ff : g.top;
            act[slot * g.ffp + u - slot * g.ff] = cw[slot] * dense_silu(gate) * upv;
        }
    }
}

// dst[n] += sum over the chosen experts of W_down act, plus the shared one.  A wave takes output rows; the experts' rows are walked as one long row, whose
// 16-byte pieces a table in LDS locates.
__global__ __launch_bounds__(512) void moe_down_step_kernel(cq_moe g, const float *__restrict__ act, const int32_t *__restrict__ ids, float *dst, const float *add, int n) {
    extern __shared__ __attribute__((aligned(16))) float xs[];             // top * ffp + shared_ffp floats, then top * ffp / 8 offsets
    const int tid = threadIdx.x, lane = tid & 63, wv = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int k1 = g.top * g.ffp, k2 = g.shared_ff ? g.shared_ffp : 0, k = k1 + k2;
    uint32_t *at = reinterpret_cast<uint32_t *>(xs + k);                   // in units of 8 weights
    for (int i = tid; i < k1 / 8; i += 512) {
        const int slot = 8 * i / g.ffp;
        at[i] = (uint32_t)((ids[slot] * g.down_stride + 8 * i - slot * g.ffp) >> 3);
    }
    for (int i = tid; 4 * i < k; i += 512) {
        f32x4 v = *reinterpret_cast<const f32x4 *>(act + 4 * i);
        const bool sh = 4 * i >= k1;
        const int c = sh ? 4 * i - k1 : 4 * i % g.ffp, ff = sh ? g.shared_ff : g.ff;
#pragma unroll
        for (int e = 0; e < 4; e++) v[e] = c + e < ff ? v[e] : 0.0f;
        reinterpret_cast<f32x4 *>(xs)[i] = v;
    }
    __syncthreads();
    const int step = gridDim.x * 8;
    constexpr int U = 8;
    for (int r = blockIdx.x * 8 + wv; r < n; r += step) {
        float acc[2] = {0.0f, 0.0f};
        const u32x4 *w = (const u32x4 *)g.down_dev + (int64_t)r * (g.ffp >> 3);
        for (int c0 = 0; c0 < k1; c0 += 512 * U) {
            u32x4 d[U];
#pragma unroll
            for (int i = 0; i < U; i++) d[i] = __builtin_nontemporal_load(w + at[min(c0 + 512 * i + 8 * lane, k1 - 8) >> 3]);
#pragma unroll
            for (int i = 0; i < U; i++) {
                const int c = c0 + 512 * i + 8 * lane;
                if (c < k1) dot8(d[i], *reinterpret_cast<const f32x4 *>(xs + c), *reinterpret_cast<const f32x4 *>(xs + c + 4), acc);
            }
        }
        const uint16_t *ws = (const uint16_t *)g.shared_down_dev + (int64_t)r * g.shared_ffp;
        for (int c0 = 0; c0 < k2; c0 += 512 * U) {
            u32x4 d[U];
#pragma unroll
            for (int i = 0; i < U; i++) d[i] = __builtin_nontemporal_load(reinterpret_cast<const u32x4 *>(ws + min(c0 + 512 * i + 8 * lane, k2 - 8)));
#pragma unroll
            for (int i = 0; i < U; i++) {
                const int c = c0 + 512 * i + 8 * lane;
                if (c < k2) dot8(d[i], *reinterpret_cast<const f32x4 *>(xs + k1 + c), *reinterpret_cast<const f32x4 *>(xs + k1 + c + 4), acc);
            }
        }
        const float s = wave_sum(acc[0] + acc[1]);
        if (lane == 0) dst[r] = dst[r] + s + (add ? add[r] : 0.0f);
    }
}

size_t up_lds(const cq_moe &g) { return (size_t)((g.kp + UP_BLOCK - 1) / UP_BLOCK) * UP_BLOCK * sizeof(float); }
size_t down_lds(const cq_moe &g) {
    const size_t k1 = (size_t)g.top * g.ffp;
    return (k1 + (g.shared_ff ? g.shared_ffp : 0)) * sizeof(float) + k1 / 8 * sizeof(uint32_t);
}
constexpr size_t STEP_LDS = 160 * 1024 - 4096;

int check_moe(const cq_moe *g) {
    if (!g) return CQ_ERR_NULL;
    if (g->experts < 1 || g->top < 1 || g->top > g->experts || g->ff < 1 || g->ffp < g->ff || g->ffp % 64 || g->kp < 64 || g->kp % 64 || g->shared_ff < 0 ||
        (g->shared_ff && (g->shared_ffp < g->shared_ff || g->shared_ffp % 64)) || g->up_stride < (int64_t)2 * g->ff * g->kp || g->up_stride % 8 || g->down_stride % 8)
        return CQ_ERR_SHAPE;
    if (g->experts > MAX_EXPERTS || g->top > MAX_TOP) return CQ_ERR_RANGE;
    return CQ_OK;
}

}  // namespace

extern "C" {

int cq_mix_moe_select(const float *logits_dev, int64_t ld, int64_t rows, int64_t experts, int64_t top, int32_t *ids_dev, float *weights_dev, float *shared_weights_dev,
                      void *stream) {
    if (rows < 0 || experts < 1 || top < 1 || top > experts || ld < experts + (shared_weights_dev ? 1 : 0)) return CQ_ERR_SHAPE;
    if (experts > MAX_EXPERTS || top > MAX_TOP || rows > (1 << 24)) return CQ_ERR_RANGE;
    if (rows == 0) return CQ_OK;
    if (!logits_dev || !ids_dev || !weights_dev) return CQ_ERR_NULL;
    hipLaunchKernelGGL(moe_select_kernel, dim3((unsigned)((rows + 3) / 4)), dim3(256), 0, (hipStream_t)stream, logits_dev, ld, rows, (int)experts, (int)top,
                       shared_weights_dev ? 1 : 0, ids_dev, weights_dev, shared_weights_dev);
    return (int)hipGetLastError();
}

int64_t cq_mix_moe_max_tiles(int64_t rows, int64_t experts, int64_t top, int64_t tile_rows) {
    if (rows < 0 || experts < 1 || top < 1 || tile_rows < 1) return -1;
    const int64_t pairs = rows * top, busy = pairs < experts ? pairs : experts;
    return pairs / tile_rows + busy;
}

int cq_mix_moe_plan(const int32_t *ids_dev, const float *weights_dev, int64_t rows, int64_t experts, int64_t top, int64_t tile_rows, int32_t *src_rows_dev,
                    int32_t *dst_rows_dev, float *scale_dev, cq_dense_tile *tiles_dev, int32_t *n_tiles_dev, void *stream) {
    if (rows < 1 || experts < 1 || top < 1 || tile_rows < 1) return CQ_ERR_SHAPE;
    if (experts > MAX_EXPERTS || top > MAX_TOP || rows * top > (1 << 24)) return CQ_ERR_RANGE;
    if (!ids_dev || !weights_dev || !src_rows_dev || !dst_rows_dev || !scale_dev || !tiles_dev || !n_tiles_dev) return CQ_ERR_NULL;
    hipLaunchKernelGGL(moe_plan_kernel, dim3(1), dim3(1024), 0, (hipStream_t)stream, ids_dev, weights_dev, (int)(rows * top), (int)experts, (int)top, (int)tile_rows,
                       src_rows_dev, dst_rows_dev, scale_dev, tiles_dev, n_tiles_dev);
    return (int)hipGetLastError();
}

int cq_mix_moe_add(const float *y_dev, int64_t ldy, int64_t top, float *x_dev, int64_t ldx, int64_t rows, int64_t dim, void *stream) {
    if (rows < 0 || top < 1 || dim < 1 || ldy % 4 || ldx % 4 || ldy < (dim + 3) / 4 * 4 || ldx < (dim + 3) / 4 * 4) return CQ_ERR_SHAPE;
    if (rows == 0) return CQ_OK;
    if (!y_dev || !x_dev) return CQ_ERR_NULL;
    if (misaligned(y_dev, 16) || misaligned(x_dev, 16)) return CQ_ERR_ALIGN;
    if (rows > 0x7fffffffLL || dim > (1 << 24)) return CQ_ERR_RANGE;
    const int64_t parts = (dim + 1023) / 1024;
    hipLaunchKernelGGL(moe_add_kernel, dim3((unsigned)rows, (unsigned)(parts < 65535 ? parts : 65535)), dim3(256), 0, (hipStream_t)stream, y_dev, ldy, (int)top, x_dev, ldx,
                       (int)dim);
    return (int)hipGetLastError();
}

int cq_mix_moe_step_fits(const cq_moe *g) {
    if (check_moe(g)) return 0;
    return up_lds(*g) <= STEP_LDS && down_lds(*g) <= STEP_LDS && (int64_t)g->experts * g->down_stride / 8 < 0xffffffffLL && (int64_t)g->top * g->ff + g->shared_ff < (1 << 30);
}

int cq_mix_moe_step(const cq_moe *g, float *x_dev, int norm, const float *vec_dev, float eps, int64_t dim, const float *logits_dev, float *act_dev, int32_t *ids_dev,
                    const float *add_dev, void *stream) {
    const int e = check_moe(g);
    if (e) return e;
    if (dim < 1 || dim > g->kp || g->down_stride < dim * (int64_t)g->ffp) return CQ_ERR_SHAPE;
    if (norm != CQ_DENSE_NORM && norm != CQ_DENSE_LAYER_NORM) return CQ_ERR_DTYPE;
    if (!x_dev || !vec_dev || !logits_dev || !act_dev || !ids_dev || !g->up_dev || !g->down_dev || (g->shared_ff && (!g->shared_up_dev || !g->shared_down_dev)))
        return CQ_ERR_NULL;
    if (misaligned(x_dev, 16) || misaligned(act_dev, 16) || misaligned(g->up_dev, 16) || misaligned(g->down_dev, 16) || misaligned(g->shared_up_dev, 16) ||
        misaligned(g->shared_down_dev, 16))
        return CQ_ERR_ALIGN;
    if (!cq_mix_moe_step_fits(g)) return CQ_ERR_RANGE;
    const size_t l1 = up_lds(*g), l2 = down_lds(*g);
    const void *up = norm == CQ_DENSE_LAYER_NORM ? reinterpret_cast<const void *>(moe_up_step_kernel<CQ_DENSE_LAYER_NORM>)
                                                 : reinterpret_cast<const void *>(moe_up_step_kernel<CQ_DENSE_NORM>);
    if (l1 > 60 * 1024) {
        const int r = (int)hipFuncSetAttribute(up, hipFuncAttributeMaxDynamicSharedMemorySize, (int)STEP_LDS);
        if (r) return r;
    }
    if (l2 > 64 * 1024) {
        const int r = (int)hipFuncSetAttribute(reinterpret_cast<const void *>(moe_down_step_kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)STEP_LDS);
        if (r) return r;
    }
    hipStream_t s = (hipStream_t)stream;
    const int64_t pairs = (int64_t)g->top * g->ff + g->shared_ff, b1 = (pairs + 7) / 8, b2 = (dim + 7) / 8;
    const dim3 grid((unsigned)(b1 < 512 ? b1 : 512));
    if (norm == CQ_DENSE_LAYER_NORM)
        hipLaunchKernelGGL(moe_up_step_kernel<CQ_DENSE_LAYER_NORM>, grid, dim3(512), l1, s, *g, x_dev, vec_dev, eps, (int)dim, logits_dev, act_dev, ids_dev);
    else
        hipLaunchKernelGGL(moe_up_step_kernel<CQ_DENSE_NORM>, grid, dim3(512), l1, s, *g, x_dev, vec_dev, eps, (int)dim, logits_dev, act_dev, ids_dev);
    hipLaunchKernelGGL(moe_down_step_kernel, dim3((unsigned)(b2 < 512 ? b2 : 512)), dim3(512), l2, s, *g, act_dev, ids_dev, x_dev, add_dev, (int)dim);
    return (int)hipGetLastError();
}

}  // extern "C"
