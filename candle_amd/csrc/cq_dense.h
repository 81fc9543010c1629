// Device helpers shared by the kernels that read bfloat16 weights.
#pragma once
#include "cq_device.h"
#include "../../include/candle_hip_mixer.h"

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));

inline bool misaligned(const void *p, size_t a) { return (reinterpret_cast<uintptr_t>(p) & (a - 1)) != 0; }

__device__ __forceinline__ float bf_lo(uint32_t v) { return __builtin_bit_cast(float, v << 16); }
__device__ __forceinline__ float bf_hi(uint32_t v) { return __builtin_bit_cast(float, v & 0xffff0000u); }

// Workgroups are dealt to the eight XCDs round-robin: give each XCD a contiguous run of tiles, so that the rows and columns
// its workgroups share stay in its own L2.
__device__ __forceinline__ int xcd_tile(int id, int total) {
    const int q = total >> 3, r = total & 7, x = id & 7, i = id >> 3;
    return x * q + min(x, r) + i;
}

__device__ __forceinline__ float dense_silu(float z) { return z / (1.0f + expf(-z)); }

// eight bf16 weights times eight f32 inputs, onto two accumulators
__device__ __forceinline__ void dot8(const u32x4 &q, const f32x4 &a, const f32x4 &b, float (&acc)[2]) {
    acc[0] = fmaf(bf_lo(q.x), a.x, acc[0]);
    acc[1] = fmaf(bf_hi(q.x), a.y, acc[1]);
    acc[0] = fmaf(bf_lo(q.y), a.z, acc[0]);
    acc[1] = fmaf(bf_hi(q.y), a.w, acc[1]);
    acc[0] = fmaf(bf_lo(q.z), b.x, acc[0]);
    acc[1] = fmaf(bf_hi(q.z), b.y, acc[1]);
    acc[0] = fmaf(bf_lo(q.w), b.z, acc[0]);
    acc[1] = fmaf(bf_hi(q.w), b.w, acc[1]);
}

// sum over a workgroup of 512 threads, in every thread (red: 8 floats)
__device__ __forceinline__ float block_sum_512(float v, float *red) {
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    return ((red[0] + red[1]) + (red[2] + red[3])) + ((red[4] + red[5]) + (red[6] + red[7]));
}

// Layer norm of a row that 512 threads have staged in LDS (zero beyond dim); vec: weight, then bias.  `sum`: the thread's share of the row's sum.
__device__ __forceinline__ void layer_norm_lds_512(float *xs, int dim, float sum, const float *__restrict__ vec, float eps, float *red) {
    const float mean = block_sum_512(sum, red) / (float)dim;
    float q = 0.0f;
    for (int i = threadIdx.x; i < dim; i += 512) {
        const float d = xs[i] - mean;
        q = fmaf(d, d, q);
    }
    const float m = sqrtf(block_sum_512(q, red) / (float)dim + eps);
    for (int i = threadIdx.x; i < dim; i += 512) xs[i] = (xs[i] - mean) / m * vec[i] + vec[dim + i];
}
