// Softmax attention whose scores are mixed across heads before the softmax, over a sliding window plus the first tokens of
// the sequence.  Mixing couples the heads, so one workgroup holds the scores of all heads for its queries and keys.
// f32 throughout (v_mfma_f32_16x16x4): scores, weights, caches.
#include "cq_mix.h"

namespace {

// A load from a wave-uniform base with a 32-bit byte offset: the address costs one register per lane.
template <typename T> __device__ __forceinline__ T ld_at(const float *base, uint32_t bytes) {
    return *reinterpret_cast<const T *>(reinterpret_cast<const char *>(base) + bytes);
}

// ---- several queries ------------------------------------------------------------------------------------------------------
// Workgroup: 16 query rows x all heads, NW waves, keys in tiles of KT, one pass with a running maximum.  Per tile:
//   scores   wave w takes heads [w NHW, (w + 1) NHW): q k^T into LDS, [head][query][key]
//   mixing   wave w takes 16 / NW queries of every head: talk x scores on the matrix cores (heads are the contracted
//            dimension), mask, running softmax in registers, weights back into the same LDS words, rescale factors to `alpha`
//   values   wave w takes U units (head, 64 output columns): weights x V added to the outputs it holds in registers, V read once per VS units
// blockIdx.y: units beyond NW U (the scores are computed again there).  blockIdx.z: split of the key tiles, for calls with too few
// query rows to fill the chip; a split leaves unnormalized outputs with their maximum and sum, talk_combine_kernel merges them.
// LDS strides: query rows of KT + 4 floats (16 rows x 4 keys of an operand read fall on 64 banks), head blocks of 16 rows + 16
// (4 heads x 16 keys likewise).
template <int NW, int NHW, bool SHARED_K, int U, int VS, int KT>
__global__ __launch_bounds__(64 * NW) void talk_attention_kernel(const float *__restrict__ q, const float *__restrict__ k_cache, const float *__restrict__ v_cache,
                                                             const float *__restrict__ talk, float scale, int window, int keep_first, float out_scale,
                                                             float *__restrict__ out, int64_t out_stride, float *__restrict__ part, int pos, int rows, int H, int G,
                                                             int dp, int vdim, int vp, int ctx) {
    constexpr int NHT = (NW * NHW + 15) / 16, HP = 16 * NHT, NT = 64 * NW, RW = 16 / NW;       // heads padded to tiles of 16; queries per wave
    constexpr int RS = KT + 4, HS = 16 * RS + 16, TS = HP + 4, KTL = KT / 16;
    extern __shared__ __attribute__((aligned(16))) float smem[];
    float *S = smem, *T = S + HP * HS, *alpha = T + HP * TS, *m_run = alpha + HP * 16, *l_run = m_run + HP * 16;      // the last three: [head][query]
    const int tid = threadIdx.x, lane = tid & 63, wv = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lk = lane >> 4;
    const int r0 = blockIdx.x * 16, nr = min(16, rows - r0);
    const int p0 = pos + r0, last = p0 + nr - 1;                         // positions of the first and last query
    const int R = H / G, nvc = (vp + 63) / 64;

    for (int i = tid; i < HP * HP; i += NT) {
        const int h = i / HP, g = i - h * HP;
        T[h * TS + g] = h < H && g < H ? talk[h * H + g] * scale : 0.0f;
    }
    for (int i = tid; i < (HP - H) * HS; i += NT) S[H * HS + i] = 0.0f;

    for (int i = tid; i < HP * 16; i += NT) {
        m_run[i] = -INFINITY;
        l_run[i] = 0.0f;
    }
    __syncthreads();
    f32x4 o[U][4];
#pragma unroll
    for (int u = 0; u < U; u++)
#pragma unroll
        for (int n = 0; n < 4; n++) o[u][n] = f32x4{0.f, 0.f, 0.f, 0.f};

    const int h0 = wv * NHW;
    const float *qb = q + (int64_t)r0 * H * dp;
    const uint32_t q_at = (min(lr, nr - 1) * H * dp + 4 * lk) * 4;
    const int u0 = ((int)blockIdx.y * NW + wv) * U, n_units = H * nvc;

    // tiles of the kept first tokens, then of the window
    const int t_lo = max(0, p0 - window + 1) / KT, t_hi = last / KT;
    const int n_keep = min((keep_first + KT - 1) / KT, t_lo);
    const int n_tiles = n_keep + t_hi - t_lo + 1, nz = gridDim.z, z = blockIdx.z;
    for (int it = n_tiles * z / nz; it < n_tiles * (z + 1) / nz; it++) {
        const int j0 = (it < n_keep ? it : t_lo + it - n_keep) * KT;
        // ---- scores ----
        if (h0 < H) {
            f32x4 acc[NHW][KTL];
#pragma unroll
            for (int i = 0; i < NHW; i++)
#pragma unroll
                for (int t = 0; t < KTL; t++) acc[i][t] = f32x4{0.f, 0.f, 0.f, 0.f};
            uint32_t k_at[KTL];
#pragma unroll
            for (int t = 0; t < KTL; t++) k_at[t] = (min(j0 + 16 * t + lr, last) * dp + 4 * lk) * 4u;
            const int64_t kv_stride = (int64_t)ctx * dp;
            for (int c = 0; c < dp; c += 16) {
                f32x4 kf[KTL], qf[NHW];
                if (SHARED_K) {
#pragma unroll
                    for (int t = 0; t < KTL; t++) kf[t] = ld_at<f32x4>(k_cache + (h0 / R) * kv_stride + c, k_at[t]);
                }
#pragma unroll
                for (int i = 0; i < NHW; i++) qf[i] = ld_at<f32x4>(qb + min(h0 + i, H - 1) * dp + c, q_at);
#pragma unroll
                for (int i = 0; i < NHW; i++) {
                    if (!SHARED_K) {
#pragma unroll
                        for (int t = 0; t < KTL; t++) kf[t] = ld_at<f32x4>(k_cache + (min(h0 + i, H - 1) / R) * kv_stride + c, k_at[t]);
                    }
#pragma unroll
                    for (int e = 0; e < 4; e++)
#pragma unroll
                        for (int t = 0; t < KTL; t++) acc[i][t] = mfma4(qf[i][e], kf[t][e], acc[i][t]);
                }
            }
#pragma unroll
            for (int i = 0; i < NHW; i++)
                if (h0 + i < H) {
#pragma unroll
                    for (int t = 0; t < KTL; t++)
#pragma unroll
                        for (int e = 0; e < 4; e++) S[(h0 + i) * HS + (4 * lk + e) * RS + 16 * t + lr] = acc[i][t][e];
                }
        }
        __syncthreads();

        // ---- mixing and softmax: queries RW wv .., one after the other ----
#pragma unroll
        for (int a = 0; a < RW; a++) {
            f32x4 acc[KTL][NHT];
#pragma unroll
            for (int t = 0; t < KTL; t++)
#pragma unroll
                for (int b = 0; b < NHT; b++) acc[t][b] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
            for (int s = 0; s < HP / 4; s++) {
                float tf[NHT], sf[KTL];
#pragma unroll
                for (int b = 0; b < NHT; b++) tf[b] = T[(16 * b + lr) * TS + 4 * s + lk];
#pragma unroll
                for (int t = 0; t < KTL; t++) sf[t] = S[(4 * s + lk) * HS + (RW * wv + a) * RS + 16 * t + lr];
#pragma unroll
                for (int t = 0; t < KTL; t++)
#pragma unroll
                    for (int b = 0; b < NHT; b++) acc[t][b] = mfma4(tf[b], sf[t], acc[t][b]);
            }
            const int p = p0 + RW * wv + a;
            bool vis[KTL];
#pragma unroll
            for (int t = 0; t < KTL; t++) {
                const int j = j0 + 16 * t + lr;
                vis[t] = j <= p && (p - j < window || j < keep_first);
            }
#pragma unroll
            for (int b = 0; b < NHT; b++)
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    float s[KTL], mx = -INFINITY, sum = 0.0f;
#pragma unroll
                    for (int t = 0; t < KTL; t++) {
                        s[t] = vis[t] ? acc[t][b][e] : -INFINITY;
                        mx = fmaxf(mx, s[t]);
                    }
                    const int h = 16 * b + 4 * lk + e, hr = h * 16 + RW * wv + a;
                    const float m_old = m_run[hr], m = fmaxf(m_old, row16_max(mx));
                    const float al = m_old > -INFINITY ? __expf(m_old - m) : 0.0f;
#pragma unroll
                    for (int t = 0; t < KTL; t++) {
                        const float w = vis[t] ? __expf(s[t] - m) : 0.0f;
                        sum += w;
                        S[h * HS + (RW * wv + a) * RS + 16 * t + lr] = w;
                    }
                    sum = row16_sum(sum);
                    m_run[hr] = m;                       // the same value from 16 lanes
                    l_run[hr] = l_run[hr] * al + sum;
                    alpha[hr] = al;
                }
        }
        __syncthreads();

        // ---- values (units beyond the last repeat it and are not stored) ----
        if (u0 < n_units) {
#pragma unroll
            for (int ub = 0; ub < U; ub += VS) {
                const int uc = min(u0 + ub, n_units - VS);
                const int g = uc / (R * nvc), c = (uc / R) % nvc, h0v = g * R + uc % R;
                const float *vb = v_cache + (int64_t)g * ctx * vp + 64 * c;
#pragma unroll
                for (int half = 0; half < KTL; half++) {
                    float vf[4][4];
#pragma unroll
                    for (int s = 0; s < 4; s++) {
                        const uint32_t at = min(j0 + 16 * half + 4 * s + lk, last) * vp;
#pragma unroll
                        for (int n = 0; n < 4; n++) vf[s][n] = ld_at<float>(vb, (at + min(16 * n + lr, vp - 64 * c - 1)) * 4u);
                    }
#pragma unroll
                    for (int v = 0; v < VS; v++) {
                        const int u = ub + v, h = h0v + v;
                        if (half == 0) {
                            const f32x4 al = *reinterpret_cast<const f32x4 *>(&alpha[h * 16 + 4 * lk]);
#pragma unroll
                            for (int n = 0; n < 4; n++) o[u][n] *= al;
                        }
#pragma unroll
                        for (int s = 0; s < 4; s++) {
                            const float w = S[h * HS + lr * RS + 16 * half + 4 * s + lk];
#pragma unroll
                            for (int n = 0; n < 4; n++) o[u][n] = mfma4(w, vf[s][n], o[u][n]);
                        }
                    }
                }
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int u = 0; u < U; u++) {
        if (u0 + u >= n_units) continue;
        const int g = (u0 + u) / (R * nvc), c = ((u0 + u) / R) % nvc, h = g * R + (u0 + u) % R;
#pragma unroll
        for (int n = 0; n < 4; n++) {
            const int col = 64 * c + 16 * n + lr;
            if (col >= vdim) continue;
#pragma unroll
            for (int e = 0; e < 4; e++) {
                const int row = 4 * lk + e;
                if (row >= nr) continue;
                if (nz == 1) out[(int64_t)(r0 + row) * out_stride + (int64_t)h * vdim + col] = out_scale * o[u][n][e] / l_run[h * 16 + row];
                else part[((int64_t)(z * rows + r0 + row) * H + h) * vdim + col] = o[u][n][e];
            }
        }
    }
    if (nz > 1 && blockIdx.y == 0) {
        float *ml = part + (int64_t)nz * rows * H * vdim;                 // [split][row][head] of (m, l)
        for (int i = tid; i < nr * H; i += NT) {
            const int row = i / H, h = i - row * H;
            float *x = ml + 2 * ((int64_t)(z * rows + r0 + row) * H + h);
            x[0] = m_run[h * 16 + row];
            x[1] = l_run[h * 16 + row];
        }
    }
}

// one wave per (row, head)
__global__ __launch_bounds__(256) void talk_combine_kernel(const float *__restrict__ part, int nz, int64_t rows, int H, int vdim, float out_scale,
                                                           float *__restrict__ out, int64_t out_stride) {
    const int lane = threadIdx.x & 63, h = blockIdx.y * 4 + (threadIdx.x >> 6);
    if (h >= H) return;
    const int64_t r = blockIdx.x, id = r * H + h, n = rows * H;
    const float *ml = part + nz * n * vdim + 2 * id;
    float m = -INFINITY, l = 0.0f;
    for (int z = 0; z < nz; z++) m = fmaxf(m, ml[2 * n * z]);
    for (int z = 0; z < nz; z++) l = fmaf(ml[2 * n * z] > -INFINITY ? __expf(ml[2 * n * z] - m) : 0.0f, ml[2 * n * z + 1], l);
    float *o = out + r * out_stride + (int64_t)h * vdim;
    for (int e = lane; e < vdim; e += 64) {
        float a = 0.0f;
        for (int z = 0; z < nz; z++) {
            const float w = ml[2 * n * z] > -INFINITY ? __expf(ml[2 * n * z] - m) : 0.0f;
            a = fmaf(w, part[(n * z + id) * vdim + e], a);
        }
        o[e] = out_scale * a / l;
    }
}

// Splits of the key tiles: as many as bring the launch to one workgroup per CU, each with at least four tiles of keys.
int talk_key_splits(int64_t rows, int64_t unit_blocks, int64_t max_keys) {
    const int64_t wg = (rows + 15) / 16 * unit_blocks, tiles = max_keys / 32;
    int64_t n = 256 / wg;
    n = n < tiles / 4 ? n : tiles / 4;
    return (int)(n < 1 ? 1 : (n > 16 ? 16 : n));
}
int talk_unit_blocks(int64_t H, int64_t vp) {               // units a launch takes: NW * U of the instance for H heads
    const int64_t per = H <= 8 ? 16 : (H <= 16 ? 32 : 64);
    return (int)((H * ((vp + 63) / 64) + per - 1) / per);
}

template <int NW, int NHW, bool SHARED_K, int U, int VS, int KT>
int talk_launch(const float *q, const float *kc, const float *vc, const float *talk, float scale, int window, int keep, float out_scale, float *out,
                int64_t out_stride, float *part, int nz, int pos, int rows, int H, int G, int dp, int vdim, int vp, int ctx, hipStream_t s) {
    constexpr int HP = (NW * NHW + 15) / 16 * 16;
    constexpr size_t lds = (size_t)(HP * (16 * (KT + 4) + 16) + HP * (HP + 4) + 3 * HP * 16) * sizeof(float);
    if (lds > 64 * 1024) {
        const int e = (int)hipFuncSetAttribute(reinterpret_cast<const void *>(talk_attention_kernel<NW, NHW, SHARED_K, U, VS, KT>),
                                               hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e) return e;
    }
    const int units = H * ((vp + 63) / 64);
    hipLaunchKernelGGL((talk_attention_kernel<NW, NHW, SHARED_K, U, VS, KT>), dim3((rows + 15) / 16, (units + NW * U - 1) / (NW * U), nz), dim3(64 * NW), lds,
                       s, q, kc, vc, talk, scale, window, keep, out_scale, out, out_stride, part, pos, rows, H, G, dp, vdim, vp, ctx);
    if (nz > 1)
        hipLaunchKernelGGL(talk_combine_kernel, dim3((unsigned)rows, (unsigned)((H + 3) / 4)), dim3(256), 0, s, (const float *)part, nz, (int64_t)rows, H, vdim, out_scale,
                           out, out_stride);
    return (int)hipGetLastError();
}

// ---- one query --------------------------------------------------------------------------------------------------------------
// Workgroup: KD of the visible keys x all heads, 16 waves.  The first K and V rows and the head mixing matrix are requested before
// anything else; meanwhile the workgroup normalizes and rotates q itself.  The one that holds the last visible key (the new token) does
// the same for k and v, appends them to the caches and uses its own copies.
//   scores  16 lanes per (kv head, key), each key row read once for the heads that share it
//   mixing  one thread per (head, key)
//   values  four lanes per (kv head, four columns), each on a quarter of the keys, four heads at a time
template <int NC, int KD>
__global__ __launch_bounds__(1024) void talk_decode_kernel(const float *__restrict__ row, cq_mix_heads gq, cq_mix_heads gk, cq_mix_heads gv, float eps,
                                                           const float *__restrict__ talk, float scale, int window, int keep_first,
                                                           const int32_t *__restrict__ pos_dev, int pos0, float *__restrict__ rec, int splits) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    const int H = gq.heads, G = gk.heads, R = H / G, dp = gk.dim_pad, vdim = gv.dim, vp = gv.dim_pad, ctx = gk.ctx;
    constexpr int SS = KD + 4, PB = 2;                               // rows of scores start on 16 bytes
    float *qs = smem, *kn = qs + H * dp, *vn = kn + G * dp, *sc = vn + G * vp, *mx = sc + H * SS, *T = mx + H * SS;
    const int tid = threadIdx.x, lane = tid & 63, wv = __builtin_amdgcn_readfirstlane(tid >> 6), sp = blockIdx.x;
    const int p = pos0 + (pos_dev ? pos_dev[0] : 0);
    const Visible vis = visible_keys(p, window, keep_first);
    const int s0 = sp * KD, cnt = min(KD, vis.n - s0);
    if (p >= ctx || cnt <= 0) return;                                // uniform: no key of this split is visible yet
    const bool owner = s0 + cnt == vis.n;                            // key cnt - 1 is the new token
    auto key_of = [&](int j) {                                       // j-th key of the split, clamped to one that exists
        const int s = s0 + min(j, cnt - 1);
        return s < vis.keep ? s : vis.lo + s - vis.keep;
    };
    const int sub = lane & 15, grp = wv * 4 + (lane >> 4), pairs = G * KD, items = G * vp / 4;
    const int quarter = tid & 3;                                     // of every 16 keys
    f32x4 kd[PB][NC], vv[4];
    auto load_k = [&](int b) {
#pragma unroll
        for (int i = 0; i < PB; i++) {
            const int pr = min(b + 64 * i, pairs - 1), g = pr / KD;
            const float *kr = gk.dst_dev + g * gk.dst_head_stride + (int64_t)key_of(pr - g * KD) * gk.dst_row_stride;
#pragma unroll
            for (int c = 0; c < NC; c++) {
                const int d = 64 * c + 4 * sub;
                kd[i][c] = d < dp ? *reinterpret_cast<const f32x4 *>(kr + d) : f32x4{0.f, 0.f, 0.f, 0.f};
            }
        }
    };
    auto load_v = [&](int i, int jb) {                               // i: four columns of a kv head
        const int g = i / (vp / 4);
        const float *vb = gv.dst_dev + g * gv.dst_head_stride + 4 * (i - g * (vp / 4));
#pragma unroll
        for (int j = 0; j < 4; j++) vv[j] = *reinterpret_cast<const f32x4 *>(vb + (int64_t)key_of(jb + 4 * quarter + j) * gv.dst_row_stride);
    };
    // Loads complete in the order they are asked for: first what the preparation needs (two query heads per wave, and for the new token
    // one head of k or v), then the mixing matrix, K and V.
    const int h2 = min(wv + 16, H - 1), xn = min(wv, 2 * G - 1);
    const cq_mix_heads &gn = xn < G ? gk : gv;
    HeadShared<NC> qsh, nsh;
    HeadRegs<NC> qa, qb, nw;
    qsh.load(gq, p, lane);
    qa.load(gq, row + gq.src_off + (int64_t)min(wv, H - 1) * gq.dim, lane);
    if (H > 16) qb.load(gq, row + gq.src_off + (int64_t)h2 * gq.dim, lane);
    if (owner) {
        nsh.load(gn, p, lane);
        nw.load(gn, row + gn.src_off + (int64_t)(xn < G ? xn : xn - G) * gn.dim, lane);
    }
    const float tv = talk[min(tid, H * H - 1)];
    load_k(grp);
    load_v(min(tid >> 2, items - 1), 0);
    qsh.ready(gq, lane);
    auto keep_q = [&](HeadRegs<NC> &x, int h) {
        x.finish(gq, qsh, eps, lane);
#pragma unroll
        for (int e = 0; e < NC; e++)
            if (h < H && lane + 64 * e < dp) qs[h * dp + lane + 64 * e] = x.v[e];
    };
    auto keep_new = [&](HeadRegs<NC> &x, int i) {
        const cq_mix_heads &gr = i < G ? gk : gv;
        const int hh = i < G ? i : i - G;
        float *dst = gr.dst_dev + hh * gr.dst_head_stride + (int64_t)p * gr.dst_row_stride, *own = (i < G ? kn : vn) + hh * gr.dim_pad;
        nsh.ready(gr, lane);
        x.finish(gr, nsh, eps, lane);
#pragma unroll
        for (int e = 0; e < NC; e++)
            if (i < 2 * G && lane + 64 * e < gr.dim_pad) dst[lane + 64 * e] = own[lane + 64 * e] = x.v[e];
    };
    keep_q(qa, wv);
    if (H > 16) keep_q(qb, wv + 16);
    if (owner && wv < 2 * G) keep_new(nw, wv);
    for (int h = wv + 32; h < H; h += 16) {
        qa.load(gq, row + gq.src_off + (int64_t)h * gq.dim, lane);
        keep_q(qa, h);
    }
    if (owner)
        for (int x = wv + 16; x < 2 * G; x += 16) {
            const cq_mix_heads &gr = x < G ? gk : gv;
            nsh.load(gr, p, lane);
            nw.load(gr, row + gr.src_off + (int64_t)(x < G ? x : x - G) * gr.dim, lane);
            keep_new(nw, x);
        }
    if (tid < H * H) T[tid] = tv * scale;
    for (int i = tid + 1024; i < H * H; i += 1024) T[i] = talk[i] * scale;
    __syncthreads();

    // ---- scores ----
    for (int b = grp; b < pairs; b += 64 * PB) {
        if (b != grp) load_k(b);
#pragma unroll
        for (int i = 0; i < PB; i++) {
            const int pr = min(b + 64 * i, pairs - 1), g = pr / KD, j = pr - g * KD;
            if (owner && j >= cnt - 1) {
#pragma unroll
                for (int c = 0; c < NC; c++)
                    if (64 * c + 4 * sub < dp) kd[i][c] = *reinterpret_cast<const f32x4 *>(kn + g * dp + 64 * c + 4 * sub);
            }
            for (int r = 0; r < R; r += 4) {                         // four heads side by side (the last one repeated)
                float a[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int c = 0; c < NC; c++) {
                    const int d = min(64 * c + 4 * sub, dp - 4);     // where dp ends, kd is zero
#pragma unroll
                    for (int x = 0; x < 4; x++) {
                        const f32x4 qv = *reinterpret_cast<const f32x4 *>(qs + (g * R + min(r + x, R - 1)) * dp + d);
                        a[x] = fmaf(qv.x, kd[i][c].x, a[x]);
                        a[x] = fmaf(qv.y, kd[i][c].y, a[x]);
                        a[x] = fmaf(qv.z, kd[i][c].z, a[x]);
                        a[x] = fmaf(qv.w, kd[i][c].w, a[x]);
                    }
                }
#pragma unroll
                for (int x = 0; x < 4; x++) a[x] = row16_sum(a[x]);
                if (sub < 4 && r + sub < R) sc[(g * R + r + sub) * SS + j] = sub == 0 ? a[0] : (sub == 1 ? a[1] : (sub == 2 ? a[2] : a[3]));
            }
        }
    }
    __syncthreads();
    // ---- mixing ----
    for (int i = tid; i < H * KD; i += 1024) {
        const int h = i / KD, j = i - h * KD;
        const float *t = T + h * H;
        float a0 = 0.0f, a1 = 0.0f;
        int g = 0;
#pragma unroll 2
        for (; g + 8 <= H; g += 8) {
            float tv8[8], sv[8];
#pragma unroll
            for (int x = 0; x < 8; x++) {
                tv8[x] = t[g + x];
                sv[x] = sc[(g + x) * SS + j];
            }
#pragma unroll
            for (int x = 0; x < 8; x += 2) {
                a0 = fmaf(tv8[x], sv[x], a0);
                a1 = fmaf(tv8[x + 1], sv[x + 1], a1);
            }
        }
        for (; g < H; g++) a0 = fmaf(t[g], sc[g * SS + j], a0);
        mx[h * SS + j] = j < cnt ? a0 + a1 : -INFINITY;
    }
    __syncthreads();
    // ---- softmax of the split: 16 lanes per head ----
    const int stride = talk_record(vdim);
    for (int h = grp; h < H; h += 64) {
        float s[KD / 16], m = -INFINITY, l = 0.0f;
#pragma unroll
        for (int i = 0; i < KD / 16; i++) {
            s[i] = mx[h * SS + 16 * i + sub];
            m = fmaxf(m, s[i]);
        }
        m = row16_max(m);
#pragma unroll
        for (int i = 0; i < KD / 16; i++) {
            s[i] = s[i] > -INFINITY ? __expf(s[i] - m) : 0.0f;
            l += s[i];
            sc[h * SS + 16 * i + sub] = s[i];
        }
        l = row16_sum(l);
        if (sub == 0) {
            float *r = rec + ((int64_t)h * splits + sp) * stride + stride - 4;
            r[0] = m;
            r[1] = l;
        }
    }
    __syncthreads();
    // ---- values ----
    const int v4 = (vdim + 3) / 4;
    for (int i = tid >> 2; i < items; i += 256) {
        const int g = i / (vp / 4), e4 = i - g * (vp / 4);
        for (int r = 0; r < R; r += 4) {
            f32x4 a[4];
#pragma unroll
            for (int x = 0; x < 4; x++) a[x] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 1
            for (int jb = 0; jb < KD; jb += 16) {
                if (i != (tid >> 2) || jb > 0 || (KD > 16 && r > 0)) load_v(i, jb);
                if (owner) {
                    const f32x4 x = *reinterpret_cast<const f32x4 *>(vn + g * vp + 4 * e4);
#pragma unroll
                    for (int j = 0; j < 4; j++)
                        if (jb + 4 * quarter + j >= cnt - 1) vv[j] = x;
                }
#pragma unroll
                for (int x = 0; x < 4; x++) {
                    const f32x4 w = *reinterpret_cast<const f32x4 *>(sc + (g * R + min(r + x, R - 1)) * SS + jb + 4 * quarter);
#pragma unroll
                    for (int j = 0; j < 4; j++)
#pragma unroll
                        for (int e = 0; e < 4; e++) a[x][e] = fmaf(w[j], vv[j][e], a[x][e]);
                }
            }
            // the sum of the four quarters in every lane; lane `quarter` stores head r + quarter
            f32x4 mine = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int x = 0; x < 4; x++)
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    const float s = quad_sum_f(a[x][e]);
                    mine[e] = quarter == x ? s : mine[e];
                }
            if (e4 < v4 && r + quarter < R) *reinterpret_cast<f32x4 *>(rec + ((int64_t)(g * R + r + quarter) * splits + sp) * stride + 4 * e4) = mine;
        }
    }
}

template <int NC, int KD>
int talk_decode_launch(const float *row, const cq_mix_heads *g, float eps, const float *talk, float scale, int window, int keep, const int32_t *pos_dev, int pos,
                       float *rec, int splits, hipStream_t s) {
    const int H = g[0].heads, G = g[1].heads;
    const size_t lds = (size_t)(H * (g[1].dim_pad + 2 * (KD + 4) + H) + G * (g[1].dim_pad + g[2].dim_pad)) * sizeof(float);
    if (lds > 160 * 1024) return CQ_ERR_RANGE;
    if (lds > 64 * 1024) {
        const int e = (int)hipFuncSetAttribute(reinterpret_cast<const void *>(talk_decode_kernel<NC, KD>), hipFuncAttributeMaxDynamicSharedMemorySize,
                                               160 * 1024);
        if (e) return e;
    }
    hipLaunchKernelGGL((talk_decode_kernel<NC, KD>), dim3(splits), dim3(1024), lds, s, row, g[0], g[1], g[2], eps, talk, scale, window, keep, pos_dev, pos, rec,
                       splits);
    return (int)hipGetLastError();
}

}  // namespace

extern "C" {

int64_t cq_mix_talk_attention_workspace_bytes(int64_t rows, int64_t n_head, int64_t vdim, int64_t window, int64_t keep_first, int64_t pos) {
    if (rows <= 0 || n_head <= 0 || vdim <= 0 || window < 1 || keep_first < 0 || pos < 0) return 0;
    const int nz = talk_key_splits(rows, talk_unit_blocks(n_head, (vdim + 15) / 16 * 16), talk_max_keys(window, keep_first, pos + rows));
    return nz > 1 ? nz * rows * n_head * (vdim + 2) * 4 : 0;
}

int cq_mix_talk_attention(const float *q_dev, const float *k_cache_dev, const float *v_cache_dev, const float *talk_dev, float scale, int64_t window,
                          int64_t keep_first, float out_scale, float *out_dev, int64_t out_stride, int64_t pos, int64_t rows, int64_t n_head,
                          int64_t n_kv_head, int64_t dim_pad, int64_t vdim, int64_t vdim_pad, int64_t ctx, void *workspace_dev, int64_t workspace_bytes, void *stream) {
    if (rows < 0 || pos < 0 || n_head <= 0 || n_kv_head <= 0 || n_head % n_kv_head || dim_pad <= 0 || dim_pad % 16 || vdim <= 0 || 
        vdim_pad != (vdim + 15) / 16 * 16 || ctx <= 0 || window < 1 || keep_first < 0 || out_stride < n_head * vdim)
        return CQ_ERR_SHAPE;
    if (rows == 0) return CQ_OK;
    if (!q_dev || !k_cache_dev || !v_cache_dev || !talk_dev || !out_dev) return CQ_ERR_NULL;
    if (mix_misaligned(q_dev, 16) || mix_misaligned(k_cache_dev, 16) || mix_misaligned(v_cache_dev, 16)) return CQ_ERR_ALIGN;
    if (pos + rows > ctx || ctx > (1 << 28) || n_head > CQ_MIX_MAX_HEADS || dim_pad > CQ_MIX_MAX_DIM || vdim_pad > CQ_MIX_MAX_DIM) return CQ_ERR_RANGE;
    if (ctx * (dim_pad > vdim_pad ? dim_pad : vdim_pad) * 4 > 0x7fffffffLL) return CQ_ERR_RANGE;      // byte offsets inside a kv head are 32-bit
    const int w = (int)(window < ctx ? window : ctx), keep = (int)(keep_first < ctx ? keep_first : ctx);
    const int H = (int)n_head, G = (int)n_kv_head, R = H / G;
    const int nz = talk_key_splits(rows, talk_unit_blocks(n_head, vdim_pad), talk_max_keys(window, keep_first, pos + rows));
    if (nz > 1 && (!workspace_dev || workspace_bytes < cq_mix_talk_attention_workspace_bytes(rows, n_head, vdim, window, keep_first, pos))) return CQ_ERR_WORKSPACE;
    hipStream_t s = (hipStream_t)stream;
#define CQ_TA(NW_, NHW_, SH_, U_, VS_, KT_)                                                                                                            \
    talk_launch<NW_, NHW_, SH_, U_, VS_, KT_>(q_dev, k_cache_dev, v_cache_dev, talk_dev, scale, w, keep, out_scale, out_dev, out_stride,      \
                                              (float *)workspace_dev, nz, (int)pos, (int)rows, H, G, (int)dim_pad, (int)vdim, (int)vdim_pad, (int)ctx, s)
    if (H <= 8) return R % 2 ? CQ_TA(8, 1, true, 2, 1, 32) : CQ_TA(8, 1, true, 2, 2, 32);
    if (H <= 16) return R % 2 ? CQ_TA(16, 1, true, 2, 1, 32) : CQ_TA(16, 1, true, 2, 2, 32);
    if (H <= 32) return R % 2 ? CQ_TA(16, 2, false, 4, 1, 32) : (R % 4 ? CQ_TA(16, 2, true, 4, 2, 32) : CQ_TA(16, 2, true, 4, 4, 32));
    return R % 4 ? CQ_TA(16, 4, false, 4, 1, 16) : CQ_TA(16, 4, true, 4, 4, 16);
#undef CQ_TA
}

int64_t cq_mix_talk_decode_workspace_bytes(int64_t n_head, int64_t vdim, int64_t window, int64_t keep_first, int64_t ctx) {
    if (n_head <= 0 || vdim <= 0 || window < 1 || keep_first < 0 || ctx <= 0) return -1;
    return n_head * talk_splits(talk_max_keys(window, keep_first, ctx)) * talk_record((int)vdim) * 4;
}

int cq_mix_talk_decode(const float *row_dev, const cq_mix_heads *qkv, float eps, const float *talk_dev, float scale, int64_t window, int64_t keep_first,
                       const int32_t *pos_dev, int64_t pos, void *workspace_dev, int64_t workspace_bytes, void *stream) {
    if (!row_dev || !qkv || !talk_dev || !workspace_dev) return CQ_ERR_NULL;
    const cq_mix_heads &q = qkv[0], &k = qkv[1], &v = qkv[2];
    for (int i = 0; i < 3; i++) {
        const int e = mix_check_group(qkv[i], i == 0);
        if (e) return e;
    }
    if (q.heads % k.heads || v.heads != k.heads || q.dim != k.dim || !k.by_position || !v.by_position || k.ctx != v.ctx || k.dim_pad % 16 || v.dim_pad % 16 ||
        window < 1 || keep_first < 0 || pos < 0 || k.dst_row_stride % 4 || k.dst_head_stride % 4 ||
        v.dst_row_stride % 4 || v.dst_head_stride % 4)
        return CQ_ERR_SHAPE;
    if (mix_misaligned(k.dst_dev, 16) || mix_misaligned(v.dst_dev, 16) || mix_misaligned(workspace_dev, 16)) return CQ_ERR_ALIGN;
    if (q.heads > CQ_MIX_MAX_HEADS || k.dim_pad > CQ_MIX_MAX_DIM || v.dim_pad > CQ_MIX_MAX_DIM || k.ctx > (1 << 28) || (!pos_dev && pos >= k.ctx)) return CQ_ERR_RANGE;
    const int64_t n_max = talk_max_keys(window, keep_first, k.ctx);
    if (workspace_bytes < cq_mix_talk_decode_workspace_bytes(q.heads, v.dim, window, keep_first, k.ctx)) return CQ_ERR_WORKSPACE;
    const int w = (int)(window < k.ctx ? window : k.ctx), keep = (int)(keep_first < k.ctx ? keep_first : k.ctx), splits = talk_splits(n_max);
    hipStream_t s = (hipStream_t)stream;
#define CQ_TD(NC_, KD_) talk_decode_launch<NC_, KD_>(row_dev, qkv, eps, talk_dev, scale, w, keep, pos_dev, (int)pos, (float *)workspace_dev, splits, s)
    const bool fine = talk_split_keys(n_max) == 16;
    const int widest = k.dim_pad > v.dim_pad ? k.dim_pad : v.dim_pad;
    if (widest <= 64) return fine ? CQ_TD(1, 16) : CQ_TD(1, 64);
    if (widest <= 128) return fine ? CQ_TD(2, 16) : CQ_TD(2, 64);
    return fine ? CQ_TD(4, 16) : CQ_TD(4, 64);
#undef CQ_TD
}

}  // extern "C"
