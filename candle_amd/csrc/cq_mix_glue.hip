// Row operations around the sequence mixers: norms of rows and heads, the normalized polynomial activation, rotation of head
// groups on their way into packed buffers and caches.
#include "cq_mix.h"

namespace {

__device__ __forceinline__ float block_sum(float v, float *red) {        // 256 threads, red: 4 floats
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    return (red[0] + red[1]) + (red[2] + red[3]);
}

template <bool VEC>
__global__ __launch_bounds__(256) void rms_norm_rows_kernel(float *x, int64_t x_stride, const int32_t *__restrict__ index, const float *__restrict__ delta,
                                                            int64_t delta_stride, const float *__restrict__ w, float *__restrict__ out,
                                                            int64_t out_stride, int dim, float eps) {
    __shared__ float red[4];
    const int64_t r = blockIdx.x;
    float *xr = x + (index ? (int64_t)index[r] : r) * x_stride;
    const float *dr = delta ? delta + r * delta_stride : nullptr;
    float *o = out + r * out_stride;
    constexpr int KEEP = 4;                        // float4 per thread kept in registers (dim <= 4096)
    if (VEC) {
        const int n4 = dim >> 2;
        f32x4 keep[KEEP];
        float acc = 0.0f;
        auto fetch = [&](int i) {
            f32x4 v = reinterpret_cast<const f32x4 *>(xr)[i];
            if (dr) {
                v += reinterpret_cast<const f32x4 *>(dr)[i];
                reinterpret_cast<f32x4 *>(xr)[i] = v;
            }
            acc = fmaf(v.x, v.x, acc);
            acc = fmaf(v.y, v.y, acc);
            acc = fmaf(v.z, v.z, acc);
            acc = fmaf(v.w, v.w, acc);
            return v;
        };
#pragma unroll
        for (int c = 0; c < KEEP; c++) {
            const int i = threadIdx.x + 256 * c;
            if (i < n4) keep[c] = fetch(i);
        }
        for (int i = threadIdx.x + 256 * KEEP; i < n4; i += 256) fetch(i);
        const float m = sqrtf(block_sum(acc, red) / (float)dim + eps);
        auto emit = [&](int i, const f32x4 &v) {
            const f32x4 a = reinterpret_cast<const f32x4 *>(w)[i];
            reinterpret_cast<f32x4 *>(o)[i] = f32x4{v.x / m * a.x, v.y / m * a.y, v.z / m * a.z, v.w / m * a.w};
        };
#pragma unroll
        for (int c = 0; c < KEEP; c++) {
            const int i = threadIdx.x + 256 * c;
            if (i < n4) emit(i, keep[c]);
        }
        for (int i = threadIdx.x + 256 * KEEP; i < n4; i += 256) emit(i, reinterpret_cast<const f32x4 *>(xr)[i]);
    } else {
        float acc = 0.0f;
        for (int i = threadIdx.x; i < dim; i += 256) {
            float v = xr[i];
            if (dr) xr[i] = v = v + dr[i];
            acc = fmaf(v, v, acc);
        }
        const float m = sqrtf(block_sum(acc, red) / (float)dim + eps);
        for (int i = threadIdx.x; i < dim; i += 256) o[i] = xr[i] / m * w[i];
    }
}

// One workgroup per row; the first KEEP * 256 values stay in registers between the mean, the variance and the result.
__global__ __launch_bounds__(256) void layer_norm_rows_kernel(const float *__restrict__ x, int64_t x_stride, const int32_t *__restrict__ index,
                                                              const float *__restrict__ vec, float *__restrict__ out, __bf16 *__restrict__ out16, int64_t out_stride, int dim,
                                                              float eps) {
    __shared__ float red[4];
    constexpr int KEEP = 16;
    const int64_t r = blockIdx.x;
    const float *xr = x + (index ? (int64_t)index[r] : r) * x_stride;
    float keep[KEEP], sum = 0.0f, q = 0.0f;
#pragma unroll
    for (int c = 0; c < KEEP; c++) {
        const int i = threadIdx.x + 256 * c;
        keep[c] = i < dim ? xr[i] : 0.0f;
        sum += keep[c];
    }
    for (int i = threadIdx.x + 256 * KEEP; i < dim; i += 256) sum += xr[i];
    const float mean = block_sum(sum, red) / (float)dim;
#pragma unroll
    for (int c = 0; c < KEEP; c++) {
        const float d = (int)threadIdx.x + 256 * c < dim ? keep[c] - mean : 0.0f;
        q = fmaf(d, d, q);
    }
    for (int i = threadIdx.x + 256 * KEEP; i < dim; i += 256) q = fmaf(xr[i] - mean, xr[i] - mean, q);
    const float m = sqrtf(block_sum(q, red) / (float)dim + eps);
    auto emit = [&](int i, float v) {
        v = (v - mean) / m * vec[i] + vec[dim + i];
        if (out) out[r * out_stride + i] = v;
        if (out16) out16[r * out_stride + i] = (__bf16)v;
    };
#pragma unroll
    for (int c = 0; c < KEEP; c++) {
        const int i = threadIdx.x + 256 * c;
        if (i < dim) emit(i, keep[c]);
    }
    for (int i = threadIdx.x + 256 * KEEP; i < dim; i += 256) emit(i, xr[i]);
}

// sum over n = 1..3 of coef[n-1] z^n / rms(z^n), plus coef[3]: one workgroup per row, the row re-read after its three sums
__global__ __launch_bounds__(256) void poly_norm_kernel(const float *z, int64_t z_stride, const float *__restrict__ coef, float *out, int64_t out_stride,
                                                        int dim, float eps) {
    __shared__ float red[4];
    const float *zr = z + (int64_t)blockIdx.x * z_stride;
    float *o = out + (int64_t)blockIdx.x * out_stride;
    float s2 = 0.0f, s4 = 0.0f, s6 = 0.0f;
    for (int i = threadIdx.x; i < dim; i += 256) {
        const float v = zr[i], q = v * v;
        s2 += q;
        s4 = fmaf(q, q, s4);
        s6 = fmaf(q * q, q, s6);
    }
    const float inv = 1.0f / (float)dim;
    const float i1 = coef[0] / sqrtf(block_sum(s2, red) * inv + eps);
    const float i2 = coef[1] / sqrtf(block_sum(s4, red) * inv + eps);
    const float i3 = coef[2] / sqrtf(block_sum(s6, red) * inv + eps);
    const float e = coef[3];
    for (int i = threadIdx.x; i < dim; i += 256) {
        const float v = zr[i], q = v * v;
        o[i] = fmaf(i1, v, fmaf(i2, q, fmaf(i3, q * v, e)));
    }
}

__global__ __launch_bounds__(256) void tanh_kernel(const float *x, int64_t x_stride, float *out, int64_t out_stride, int dim) {
    const float *xr = x + (int64_t)blockIdx.x * x_stride;
    float *o = out + (int64_t)blockIdx.x * out_stride;
    for (int i = threadIdx.x; i < dim; i += 256) o[i] = tanhf(xr[i]);
}

struct Groups {
    cq_mix_heads g[CQ_MIX_MAX_GROUPS];
};

// One wave per (row, up to PACK_HEADS heads of a group): what depends on the position is loaded once for them, and all their values are
// requested before the first is worked on.  blockIdx.x: row, blockIdx.y: four waves.
constexpr int PACK_HEADS = 8;
template <int NE>
__global__ __launch_bounds__(256) void pack_heads_kernel(const float *__restrict__ src, int64_t src_stride, Groups gs, int n_groups, float eps,
                                                         const int32_t *__restrict__ pos_dev, int64_t pos) {
    const int lane = threadIdx.x & 63;
    int c = blockIdx.y * 4 + __builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6)), gi = 0;
    while (gi < n_groups && c >= (gs.g[gi].heads + PACK_HEADS - 1) / PACK_HEADS) c -= (gs.g[gi++].heads + PACK_HEADS - 1) / PACK_HEADS;
    if (gi == n_groups) return;
    const cq_mix_heads g = gs.g[gi];
    const int64_t r = blockIdx.x, p = pos + (pos_dev ? pos_dev[0] : 0) + r;
    if (g.ctx > 0 && p >= g.ctx) return;
    const int h0 = c * PACK_HEADS;
    const float *s = src + r * src_stride + g.src_off;
    float *d = g.dst_dev + (g.by_position ? p : r) * g.dst_row_stride;
    HeadShared<NE> sh;
    HeadRegs<NE> x[PACK_HEADS];
    sh.load(g, p, lane);
#pragma unroll
    for (int i = 0; i < PACK_HEADS; i++) x[i].load(g, s + (int64_t)min(h0 + i, g.heads - 1) * g.dim, lane);
    sh.ready(g, lane);
#pragma unroll
    for (int i = 0; i < PACK_HEADS; i++) {
        x[i].finish(g, sh, eps, lane);
        if (h0 + i < g.heads)
#pragma unroll
            for (int e = 0; e < NE; e++)
                if (lane + 64 * e < g.dim_pad) d[(h0 + i) * g.dst_head_stride + lane + 64 * e] = x[i].v[e];
    }
}

__device__ __forceinline__ float gated(float v, float g, int kind) {
    const float sg = mix_sigmoid(g);
    return v * (kind == CQ_GATE_SILU ? g * sg : sg);
}

// One wave per (row, NH heads) of up to 64 NE dimensions, everything requested before the first sum.
template <int NE, int NH>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(const float *__restrict__ o, int64_t o_stride, const float *__restrict__ gate, int64_t g_stride,
                                                             const float *__restrict__ w, int kind, float scale, float *__restrict__ out, int64_t out_stride,
                                                             int heads, int dim, float eps) {
    const int lane = threadIdx.x & 63;
    const int h0 = (blockIdx.y * 4 + __builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6))) * NH;
    if (h0 >= heads) return;
    const int64_t r = blockIdx.x;
    const float *orow = o + r * o_stride, *grow = gate + r * g_stride;
    float *dst = out + r * out_stride;
    float v[NH][NE], g[NH][NE];
#pragma unroll
    for (int i = 0; i < NH; i++)
#pragma unroll
        for (int e = 0; e < NE; e++) {
            const int d = lane + 64 * e, at = min(h0 + i, heads - 1) * dim + d;
            v[i][e] = d < dim ? orow[at] : 0.0f;
            g[i][e] = d < dim ? grow[at] : 0.0f;
        }
#pragma unroll
    for (int i = 0; i < NH; i++) {
        float q = 0.0f;
#pragma unroll
        for (int e = 0; e < NE; e++) q = fmaf(v[i][e], v[i][e], q);
        const float inv = 1.0f / sqrtf(wave_sum(q) / (float)dim + eps);
#pragma unroll
        for (int e = 0; e < NE; e++) {
            const int d = lane + 64 * e, at = (h0 + i) * dim + d;
            if (h0 + i < heads && d < dim) dst[at] = scale * gated(v[i][e] * inv * (w ? w[at] : 1.0f), g[i][e], kind);
        }
    }
}

// heads of any size
__global__ __launch_bounds__(256) void head_norm_gate_long_kernel(const float *__restrict__ o, int64_t o_stride, const float *__restrict__ gate, int64_t g_stride,
                                                                  const float *__restrict__ w, int kind, float scale, float *__restrict__ out,
                                                                  int64_t out_stride, int heads, int dim, float eps) {
    const int lane = threadIdx.x & 63;
    const int h = blockIdx.y * 4 + (threadIdx.x >> 6);
    if (h >= heads) return;
    const int64_t r = blockIdx.x, hd = (int64_t)h * dim;
    const float *s = o + r * o_stride + hd;
    const float inv = head_inv_rms(s, dim, eps, lane);
    for (int i = lane; i < dim; i += 64) out[r * out_stride + hd + i] = scale * gated(s[i] * inv * (w ? w[hd + i] : 1.0f), gate[r * g_stride + hd + i], kind);
}

}  // namespace

extern "C" {

int cq_mix_rms_norm_rows(float *x_dev, int64_t x_stride, const int32_t *index_dev, const float *delta_dev, int64_t delta_stride, const float *weight_dev,
                         float *out_dev, int64_t out_stride, int64_t rows, int64_t dim, float eps, void *stream) {
    if (rows < 0 || dim <= 0 || x_stride < dim || out_stride < dim || (delta_dev && delta_stride < dim)) return CQ_ERR_SHAPE;
    if (rows == 0) return CQ_OK;
    if (!x_dev || !weight_dev || !out_dev) return CQ_ERR_NULL;
    if (index_dev && delta_dev) return CQ_ERR_SHAPE;            // selected rows are only read
    if (rows > 0x7fffffffLL || dim > (1 << 24)) return CQ_ERR_RANGE;
    const bool vec = dim % 4 == 0 && x_stride % 4 == 0 && out_stride % 4 == 0 && (!delta_dev || delta_stride % 4 == 0) && !mix_misaligned(x_dev, 16) &&
                     !mix_misaligned(delta_dev, 16) && !mix_misaligned(weight_dev, 16) && !mix_misaligned(out_dev, 16);
    hipStream_t s = (hipStream_t)stream;
    if (vec)
        hipLaunchKernelGGL(rms_norm_rows_kernel<true>, dim3((unsigned)rows), dim3(256), 0, s, x_dev, x_stride, index_dev, delta_dev, delta_stride, weight_dev,
                           out_dev, out_stride, (int)dim, eps);
    else
        hipLaunchKernelGGL(rms_norm_rows_kernel<false>, dim3((unsigned)rows), dim3(256), 0, s, x_dev, x_stride, index_dev, delta_dev, delta_stride, weight_dev,
                           out_dev, out_stride, (int)dim, eps);
    return (int)hipGetLastError();
}

int cq_mix_layer_norm_rows(const float *x_dev, int64_t x_stride, const int32_t *index_dev, const float *vec_dev, float *out_dev, void *out_bf16_dev,
                           int64_t out_stride, int64_t rows, int64_t dim, float eps, void *stream) {
    if (rows < 0 || dim <= 0 || x_stride < dim || out_stride < dim) return CQ_ERR_SHAPE;
    if (rows == 0) return CQ_OK;
    if (!x_dev || !vec_dev || (!out_dev && !out_bf16_dev)) return CQ_ERR_NULL;
    if (rows > 0x7fffffffLL || dim > (1 << 24)) return CQ_ERR_RANGE;
    hipLaunchKernelGGL(layer_norm_rows_kernel, dim3((unsigned)rows), dim3(256), 0, (hipStream_t)stream, x_dev, x_stride, index_dev, vec_dev, out_dev,
                       (__bf16 *)out_bf16_dev, out_stride, (int)dim, eps);
    return (int)hipGetLastError();
}

int cq_mix_poly_norm(const float *z_dev, int64_t z_stride, const float *coef_dev, float *out_dev, int64_t out_stride, int64_t rows, int64_t dim, float eps,
                     void *stream) {
    if (rows < 0 || dim <= 0 || z_stride < dim || out_stride < dim) return CQ_ERR_SHAPE;
    if (rows == 0) return CQ_OK;
    if (!z_dev || !coef_dev || !out_dev) return CQ_ERR_NULL;
    if (rows > 0x7fffffffLL || dim > (1 << 24)) return CQ_ERR_RANGE;
    hipLaunchKernelGGL(poly_norm_kernel, dim3((unsigned)rows), dim3(256), 0, (hipStream_t)stream, z_dev, z_stride, coef_dev, out_dev, out_stride, (int)dim, eps);
    return (int)hipGetLastError();
}

int cq_mix_tanh(const float *x_dev, int64_t x_stride, float *out_dev, int64_t out_stride, int64_t rows, int64_t dim, void *stream) {
    if (rows < 0 || dim <= 0 || x_stride < dim || out_stride < dim) return CQ_ERR_SHAPE;
    if (rows == 0) return CQ_OK;
    if (!x_dev || !out_dev) return CQ_ERR_NULL;
    if (rows > 0x7fffffffLL || dim > (1 << 24)) return CQ_ERR_RANGE;
    hipLaunchKernelGGL(tanh_kernel, dim3((unsigned)rows), dim3(256), 0, (hipStream_t)stream, x_dev, x_stride, out_dev, out_stride, (int)dim);
    return (int)hipGetLastError();
}

int cq_mix_pack_heads(const float *src_dev, int64_t src_stride, const cq_mix_heads *groups, int n_groups, float eps, const int32_t *pos_dev, int64_t pos,
                      int64_t rows, void *stream) {
    if (n_groups < 1 || n_groups > CQ_MIX_MAX_GROUPS || rows < 0 || pos < 0) return CQ_ERR_SHAPE;
    if (rows == 0) return CQ_OK;
    if (!src_dev || !groups) return CQ_ERR_NULL;
    Groups gs;
    int64_t chunks = 0;
    int widest = 0;
    for (int i = 0; i < n_groups; i++) {
        const int e = mix_check_group(groups[i], false);
        if (e) return e;
        if (groups[i].src_off + (int64_t)groups[i].heads * groups[i].dim > src_stride) return CQ_ERR_SHAPE;
        if (groups[i].ctx > 0 && !pos_dev && pos + rows > groups[i].ctx) return CQ_ERR_RANGE;
        gs.g[i] = groups[i];
        chunks += (groups[i].heads + PACK_HEADS - 1) / PACK_HEADS;
        widest = groups[i].dim_pad > widest ? groups[i].dim_pad : widest;
    }
    if (rows > 0x7fffffffLL || chunks > 4 * 65535) return CQ_ERR_RANGE;
    const dim3 grid((unsigned)rows, (unsigned)((chunks + 3) / 4));
    hipStream_t s = (hipStream_t)stream;
#define CQ_PH(NE_) hipLaunchKernelGGL(pack_heads_kernel<NE_>, grid, dim3(256), 0, s, src_dev, src_stride, gs, n_groups, eps, pos_dev, pos)
    if (widest <= 64) CQ_PH(1);
    else if (widest <= 128) CQ_PH(2);
    else CQ_PH(4);
#undef CQ_PH
    return (int)hipGetLastError();
}

int cq_mix_head_norm_gate(const float *o_dev, int64_t o_stride, const float *g_dev, int64_t g_stride, const float *weight_dev, int gate, float scale,
                          float *out_dev, int64_t out_stride, int64_t rows, int64_t heads, int64_t dim, float eps, void *stream) {
    if (rows < 0 || heads <= 0 || dim <= 0 || o_stride < heads * dim || g_stride < heads * dim || out_stride < heads * dim) return CQ_ERR_SHAPE;
    if (gate != CQ_GATE_SILU && gate != CQ_GATE_SIGMOID) return CQ_ERR_DTYPE;
    if (rows == 0) return CQ_OK;
    if (!o_dev || !g_dev || !out_dev) return CQ_ERR_NULL;
    if (heads * dim > (1 << 24) || heads > 4 * 65535 || rows > 0x7fffffffLL) return CQ_ERR_RANGE;
    hipStream_t s = (hipStream_t)stream;
#define CQ_HG(K_, NH_)                                                                                                                                 \
    hipLaunchKernelGGL(K_, dim3((unsigned)rows, (unsigned)((heads + 4 * NH_ - 1) / (4 * NH_))), dim3(256), 0, s, o_dev, o_stride, g_dev, g_stride, weight_dev, gate, \
                       scale, out_dev, out_stride, (int)heads, (int)dim, eps)
    if (dim <= 64) CQ_HG((head_norm_gate_kernel<1, 8>), 8);
    else if (dim <= 128) CQ_HG((head_norm_gate_kernel<2, 4>), 4);
    else if (dim <= 256) CQ_HG((head_norm_gate_kernel<4, 2>), 2);
    else CQ_HG(head_norm_gate_long_kernel, 1);
#undef CQ_HG
    return (int)hipGetLastError();
}

}  // extern "C"
