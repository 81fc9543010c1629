// Device helpers shared by the sequence-mixer kernels.
#pragma once
#include "cq_device.h"
#include "../../include/candle_hip_mixer.h"

inline bool mix_misaligned(const void *p, size_t a) { return (reinterpret_cast<uintptr_t>(p) & (a - 1)) != 0; }

__device__ __forceinline__ float mix_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

__device__ __forceinline__ f32x4 mfma4(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// 1 / root mean square of a head (one wave; lane takes dimensions lane, lane + 64, ...)
__device__ __forceinline__ float head_inv_rms(const float *src, int dim, float eps, int lane) {
    float s = 0.0f;
    for (int d = lane; d < dim; d += 64) s = fmaf(src[d], src[d], s);
    return 1.0f / sqrtf(wave_sum(s) / (float)dim + eps);
}

// Element `other` (0 .. 64 NE - 1, lane's own choice) of a vector that a wave holds as lane + 64 e.
template <int NE>
__device__ __forceinline__ float wave_gather(const float (&x)[NE], int other) {
    float r = 0.0f;
#pragma unroll
    for (int e = 0; e < NE; e++) {
        const float v = __shfl(x[e], other & 63, 64);
        r = (other >> 6) == e ? v : r;
    }
    return r;
}

// Heads of a group in the registers of a wave (lane: dimensions lane + 64 e).  HeadShared is what all heads of the group need at position p;
// a head itself is one load per 64 dimensions.  The vector memory pipeline takes an instruction per 16 cycles whatever it loads, so
// rotation partners come from other lanes, not from memory.
template <int NE>
struct HeadShared {
    float w[NE], wo[NE], c[NE], s[NE];           // norm weight, that of the rotation partner, cos, sin
    __device__ __forceinline__ void load(const cq_mix_heads &g, int64_t p, int lane) {
        const int half = g.rot_dims >> 1;
#pragma unroll
        for (int e = 0; e < NE; e++) {
            const int d = lane + 64 * e, i = d < half ? d : d - half;
            const bool rot = d < g.rot_dims;
            w[e] = d < g.dim && g.norm_dev ? g.norm_dev[d] : 1.0f;
            c[e] = rot ? g.cos_dev[p * half + i] : 1.0f;
            s[e] = rot ? g.sin_dev[p * half + i] : 0.0f;
        }
    }
    // after all loads have been asked for
    __device__ __forceinline__ void ready(const cq_mix_heads &g, int lane) {
        if (!g.norm_dev || !g.rot_dims) {
#pragma unroll
            for (int e = 0; e < NE; e++) wo[e] = w[e];
            return;
        }
#pragma unroll
        for (int e = 0; e < NE; e++) wo[e] = wave_gather(w, partner(g, lane + 64 * e));
    }
    static __device__ __forceinline__ int partner(const cq_mix_heads &g, int d) {
        const int half = g.rot_dims >> 1;
        return d < half ? d + half : (d < g.rot_dims ? d - half : d);
    }
};

template <int NE>
struct HeadRegs {
    float v[NE];
    __device__ __forceinline__ void load(const cq_mix_heads &g, const float *src, int lane) {
#pragma unroll
        for (int e = 0; e < NE; e++) v[e] = lane + 64 * e < g.dim ? src[lane + 64 * e] : 0.0f;
    }
    // norm, rotation and factor in place (zero beyond dim)
    __device__ __forceinline__ void finish(const cq_mix_heads &g, const HeadShared<NE> &sh, float eps, int lane) {
        float inv = 1.0f, o[NE];
        if (g.norm_dev) {
            float q = 0.0f;
#pragma unroll
            for (int e = 0; e < NE; e++) q = fmaf(v[e], v[e], q);
            inv = 1.0f / sqrtf(wave_sum(q) / (float)g.dim + eps);
        }
        const int half = g.rot_dims >> 1;
        if (half)
#pragma unroll
            for (int e = 0; e < NE; e++) o[e] = wave_gather(v, HeadShared<NE>::partner(g, lane + 64 * e));
        else
#pragma unroll
            for (int e = 0; e < NE; e++) o[e] = 0.0f;
#pragma unroll
        for (int e = 0; e < NE; e++) {
            const float a = v[e] * inv * sh.w[e], b = o[e] * inv * sh.wo[e];
            v[e] = (lane + 64 * e < half ? a * sh.c[e] - b * sh.s[e] : a * sh.c[e] + b * sh.s[e]) * g.factor;
        }
    }
};

// shapes and pointers of a group that a kernel will read (and write, unless `no_dst`)
inline int mix_check_group(const cq_mix_heads &g, bool no_dst) {
    if (g.heads <= 0 || g.dim <= 0 || g.src_off < 0 || g.rot_dims < 0 || g.rot_dims % 2 || g.rot_dims > g.dim) return CQ_ERR_SHAPE;
    if (g.dim > CQ_MIX_MAX_DIM || g.dim_pad > CQ_MIX_MAX_DIM) return CQ_ERR_RANGE;
    if (g.rot_dims && (!g.cos_dev || !g.sin_dev)) return CQ_ERR_NULL;
    if (g.rot_dims && g.ctx <= 0) return CQ_ERR_SHAPE;
    if (no_dst) return CQ_OK;
    if (!g.dst_dev) return CQ_ERR_NULL;
    if (g.dim_pad < g.dim || (g.by_position && g.ctx <= 0)) return CQ_ERR_SHAPE;
    return CQ_OK;
}

// Keys that position p sees, in order: [0, keep) then [lo, p].
struct Visible {
    int keep, lo, n;
};
__host__ __device__ inline Visible visible_keys(int p, int window, int keep_first) {
    Visible v;
    v.lo = p >= window ? p - window + 1 : 0;
    v.keep = keep_first < v.lo ? keep_first : v.lo;
    v.n = v.keep + p - v.lo + 1;
    return v;
}

// Split of a single token's visible keys over workgroups, and the record each leaves per head: acc[vdim], then m and l.
__host__ __device__ inline int64_t talk_max_keys(int64_t window, int64_t keep_first, int64_t ctx) {
    const int64_t n = keep_first > ctx - window ? ctx : window + keep_first;
    return n < ctx ? n : ctx;
}
__host__ __device__ inline int talk_split_keys(int64_t max_keys) { return max_keys <= 4096 ? 16 : 64; }
__host__ __device__ inline int talk_splits(int64_t max_keys) { return (int)((max_keys + talk_split_keys(max_keys) - 1) / talk_split_keys(max_keys)); }
__host__ __device__ inline int talk_record(int vdim) { return (vdim + 3) / 4 * 4 + 4; }

// max over each aligned group of 16 lanes, in every lane
__device__ __forceinline__ float row16_max(float v) {
#define CQ_MX(ctrl) v = fmaxf(v, __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), ctrl, 0xf, 0xf, true)))
    CQ_MX(CQ_DPP_QUAD_XOR1);
    CQ_MX(CQ_DPP_QUAD_XOR2);
    CQ_MX(CQ_DPP_ROW_HALF_MIRROR);
    CQ_MX(0x140);                                          // row_mirror
#undef CQ_MX
    return v;
}

// sum over each aligned group of 4 lanes, in every lane
__device__ __forceinline__ float quad_sum_f(float v) {
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CQ_DPP_QUAD_XOR1, 0xf, 0xf, true));
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CQ_DPP_QUAD_XOR2, 0xf, 0xf, true));
    return v;
}
