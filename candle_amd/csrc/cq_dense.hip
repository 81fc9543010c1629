// Matrix products with unquantized bfloat16 weights: MFMA tiles for several activation rows (bf16 or f32 products, f32
// accumulation), plain, batched or grouped by expert; a weight-streaming matvec for one row with the norm / activation of the
// input as prologue and the residual add as epilogue.  Activations and results are f32 in memory, like everywhere in this library
// (the bf16 product rounds them on the way into LDS), or bfloat16 where a caller feeds another bf16 product.
#include "cq_dense.h"

namespace {

__device__ __forceinline__ bf16x8 round_bf16(const f32x4 &a, const f32x4 &b) {
    bf16x8 r;
#pragma unroll
    for (int i = 0; i < 4; i++) {
        r[i] = (__bf16)a[i];
        r[4 + i] = (__bf16)b[i];
    }
    return r;
}

// where a tile's results go: the plane of a k split, or dst with the epilogue
struct Out {
    void *dst;
    const float *add;
    int64_t ldd, ld_add;
    float *planes;          // != nullptr: [splits][m][n4]
    int64_t n4;             // n rounded up to 4
    int accumulate, act, bf16;
    const float *row_scale;
    const int32_t *rows;    // row m goes to row rows[m] of dst
    int64_t batch;          // elements of dst per batch
};

// what a tile reads: weights and activations (f32 or bf16), which row of x row m is, and the group of a tile of rows
struct Src {
    const uint16_t *w;
    const void *x;
    int64_t ldw, ldx, w_batch, x_batch;
    const int32_t *rows;
    const cq_dense_tile *tiles;
    const int32_t *n_tiles;
};

__device__ __forceinline__ void put(const Out &o, int64_t at, float v) {
    if (o.bf16) reinterpret_cast<__bf16 *>(o.dst)[at] = (__bf16)v;
    else reinterpret_cast<float *>(o.dst)[at] = v;
}

// four consecutive columns n .. n+3 of row m (n % 4 == 0)
__device__ __forceinline__ void emit4(const Out &o, f32x4 v, int64_t m, int n, int64_t M, int N, int split) {
    if (o.planes) {
        *reinterpret_cast<f32x4 *>(o.planes + ((int64_t)split * M + m) * o.n4 + n) = v;
        return;
    }
    const int64_t r = o.rows ? o.rows[m] : m;
    if (o.act == CQ_DENSE_ACT_SWIGLU) {                    // columns are gate, up, gate, up
        const float sc = o.row_scale ? o.row_scale[m] : 1.0f;
        const float a = sc * dense_silu(v.x) * v.y, b = sc * dense_silu(v.z) * v.w;
        const int64_t at = r * o.ldd + (n >> 1);
        put(o, at, a);
        if (n + 3 < N) put(o, at + 1, b);
        return;
    }
    if (o.act == CQ_DENSE_ACT_RELU2) {
#pragma unroll
        for (int i = 0; i < 4; i++) v[i] = fmaxf(v[i], 0.0f) * fmaxf(v[i], 0.0f);
    }
    if (o.row_scale) v *= o.row_scale[m];
    if (o.bf16) {
        __bf16 *d = reinterpret_cast<__bf16 *>(o.dst) + r * o.ldd + n;
        if (n + 4 <= N && (reinterpret_cast<uintptr_t>(d) & 7) == 0) {
            bf16x4 b;
#pragma unroll
            for (int i = 0; i < 4; i++) b[i] = (__bf16)v[i];
            *reinterpret_cast<bf16x4 *>(d) = b;
            return;
        }
#pragma unroll
        for (int i = 0; i < 4; i++)
            if (n + i < N) d[i] = (__bf16)v[i];
        return;
    }
    float *d = reinterpret_cast<float *>(o.dst) + r * o.ldd + n;
    const float *a = o.add ? o.add + r * o.ld_add + n : nullptr;
    if (n + 4 <= N && ((reinterpret_cast<uintptr_t>(d) | reinterpret_cast<uintptr_t>(a)) & 15) == 0) {
        if (o.accumulate) v += *reinterpret_cast<const f32x4 *>(d);
        if (a) v += *reinterpret_cast<const f32x4 *>(a);
        *reinterpret_cast<f32x4 *>(d) = v;
        return;
    }
#pragma unroll
    for (int i = 0; i < 4; i++)
        if (n + i < N) d[i] = v[i] + (o.accumulate ? d[i] : 0.0f) + (a ? a[i] : 0.0f);
}

// Tile t of the order that a run follows: GROUP row tiles wide, column by column, so that the workgroups running side by side on an XCD need
// few distinct rows of either operand (f32 rows are twice the bytes of weight rows: a group narrower than it is long).  GROUP 4 / 6 / 8 / 16 at
// 4096 rows: 705 / 686-732 / 683-702 / 634-663 TFLOP/s, all row tiles first 449-474.
constexpr int TILE_GROUP = 6;
__device__ __forceinline__ void tile_at(int t, int tiles_m, int tiles_n, int &tm, int &tn) {
    const int grp = t / (TILE_GROUP * tiles_n), wide = min(TILE_GROUP, tiles_m - TILE_GROUP * grp), in = t - TILE_GROUP * grp * tiles_n;
    tm = TILE_GROUP * grp + in % wide;
    tn = in / wide;
}

// ---- bf16 tiles: BM activation rows x BN weight rows, k in steps of 64, LDS double-buffered -----------------------------
// The weights are the A operand, so a lane ends with four consecutive output columns of one row.  LDS rows are 128 bytes in
// eight 16-byte chunks, chunk c of row r at c ^ (r & 7).
// XB: the activations are bfloat16.  With a table of tiles (grouped products) the rows of a tile share the weights of one group.
template <int BM, int BN, int WGM, int WGN, bool XB>
__global__ __launch_bounds__(256, 2) void dense_bf16_kernel(Src src, Out out, int64_t M, int N, int K, int tiles_m, int tiles_n, int k_split) {
    constexpr int XV = XB ? 1 : 2;                         // 16-byte loads per eight activations
    constexpr int TM = BM / WGM / 16, TN = BN / WGN / 16, CA = BM * 8 / 256, CB = BN * 8 / 256;
    __shared__ bf16x8 lds[2][(BM + BN) * 8];
    const int tid = threadIdx.x, lane = tid & 63, wv = __builtin_amdgcn_readfirstlane(tid >> 6);
    if (src.tiles) {
        tiles_m = min(src.n_tiles[0], tiles_m);
        if ((int)blockIdx.x >= tiles_m * tiles_n) return;
    }
    int tm, tn;
    tile_at(xcd_tile(blockIdx.x, tiles_m * tiles_n), tiles_m, tiles_n, tm, tn);
    int64_t m0 = (int64_t)tm * BM;
    const uint16_t *w = src.w + blockIdx.z * src.w_batch;
    if (src.tiles) {
        const cq_dense_tile t = src.tiles[tm];
        m0 = t.first;
        M = t.first + t.rows;
        w += t.group * src.w_batch;
    }
    out.dst = out.bf16 ? (void *)(reinterpret_cast<uint16_t *>(out.dst) + blockIdx.z * out.batch) : (void *)(reinterpret_cast<float *>(out.dst) + blockIdx.z * out.batch);
    const int n0 = tn * BN;
    const int k_lo = blockIdx.y * k_split, k_hi = min(K, k_lo + k_split);
    const int wm = (wv / WGN) * (BM / WGM), wn = (wv % WGN) * (BN / WGN);

    u32x4 ra[CA][XV];
    u32x4 rb[CB];
    const uint8_t *xp[CA];                                 // row starts, in bytes
    const uint16_t *wp[CB];
#pragma unroll
    for (int i = 0; i < CA; i++) {
        const int c = tid + 256 * i;
        int64_t r = min(m0 + (c >> 3), M - 1);
        if (src.rows) r = src.rows[r];
        xp[i] = reinterpret_cast<const uint8_t *>(src.x) + (blockIdx.z * src.x_batch + r * src.ldx + (c & 7) * 8) * (XB ? 2 : 4);
    }
#pragma unroll
    for (int i = 0; i < CB; i++) {
        const int c = tid + 256 * i;
        wp[i] = w + (int64_t)min(n0 + (c >> 3), N - 1) * src.ldw + (c & 7) * 8;
    }
    auto fetch = [&](int k) {
#pragma unroll
        for (int i = 0; i < CB; i++) rb[i] = *reinterpret_cast<const u32x4 *>(wp[i] + k);
#pragma unroll
        for (int i = 0; i < CA; i++) {
#pragma unroll
            for (int j = 0; j < XV; j++) ra[i][j] = *reinterpret_cast<const u32x4 *>(xp[i] + (int64_t)k * (XB ? 2 : 4) + 16 * j);
        }
    };
    auto stage = [&](int b) {
#pragma unroll
        for (int i = 0; i < CB; i++) {
            const int c = tid + 256 * i, r = c >> 3;
            lds[b][BM * 8 + r * 8 + ((c & 7) ^ (r & 7))] = __builtin_bit_cast(bf16x8, rb[i]);
        }
#pragma unroll
        for (int i = 0; i < CA; i++) {
            const int c = tid + 256 * i, r = c >> 3;
            lds[b][r * 8 + ((c & 7) ^ (r & 7))] =
                XB ? __builtin_bit_cast(bf16x8, ra[i][0]) : round_bf16(__builtin_bit_cast(f32x4, ra[i][0]), __builtin_bit_cast(f32x4, ra[i][XV - 1]));
        }
    };
    f32x4 acc[TM][TN];
#pragma unroll
    for (int i = 0; i < TM; i++)
#pragma unroll
        for (int j = 0; j < TN; j++) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};

    fetch(k_lo);
    stage(0);
    __syncthreads();
    int cur = 0;
    const int lr = lane & 15, lk = lane >> 4;
    for (int k = k_lo; k < k_hi; k += 64) {
        const bool more = k + 64 < k_hi;
        if (more) fetch(k + 64);
#pragma unroll
        for (int s = 0; s < 2; s++) {
            bf16x8 fa[TM], fb[TN];
#pragma unroll
            for (int i = 0; i < TM; i++) {
                const int r = wm + 16 * i + lr;
                fa[i] = lds[cur][r * 8 + ((4 * s + lk) ^ (r & 7))];
            }
#pragma unroll
            for (int j = 0; j < TN; j++) {
                const int r = wn + 16 * j + lr;
                fb[j] = lds[cur][BM * 8 + r * 8 + ((4 * s + lk) ^ (r & 7))];
            }
#pragma unroll
            for (int i = 0; i < TM; i++)
#pragma unroll
                for (int j = 0; j < TN; j++) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fb[j], fa[i], acc[i][j], 0, 0, 0);
        }
        if (more) {
            stage(cur ^ 1);
            __syncthreads();
            cur ^= 1;
        }
    }
#pragma unroll
    for (int i = 0; i < TM; i++) {
        const int64_t m = m0 + wm + 16 * i + lr;
        if (m >= M) continue;
#pragma unroll
        for (int j = 0; j < TN; j++) {
            const int n = n0 + wn + 16 * j + 4 * lk;
            if (n < N) emit4(out, acc[i][j], m, n, M, N, blockIdx.y);
        }
    }
}

// ---- f32 tiles: 64 x 64, k in steps of 32, weights widened on the way into LDS; a lane's float4 along k feeds four steps of
// v_mfma_f32_16x16x4 (both operands use the same k order) ------------------------------------------------------------------
constexpr int DF_ROW = 36;               // floats per LDS row: 32 + 4, 16 rows of a 16-byte read fall on distinct banks
__global__ __launch_bounds__(256) void dense_f32_kernel(Src src, Out out, int64_t M, int N, int K, int tiles_m, int tiles_n, int k_split) {
    __shared__ float lds[2][128 * DF_ROW];
    const int tid = threadIdx.x, lane = tid & 63, wv = __builtin_amdgcn_readfirstlane(tid >> 6);
    if (src.tiles) {
        tiles_m = min(src.n_tiles[0], tiles_m);
        if ((int)blockIdx.x >= tiles_m * tiles_n) return;
    }
    int tm, tn;
    tile_at(xcd_tile(blockIdx.x, tiles_m * tiles_n), tiles_m, tiles_n, tm, tn);
    int64_t m0 = (int64_t)tm * 64;
    const uint16_t *w = src.w + blockIdx.z * src.w_batch;
    if (src.tiles) {
        const cq_dense_tile t = src.tiles[tm];
        m0 = t.first;
        M = t.first + t.rows;
        w += t.group * src.w_batch;
    }
    out.dst = out.bf16 ? (void *)(reinterpret_cast<uint16_t *>(out.dst) + blockIdx.z * out.batch) : (void *)(reinterpret_cast<float *>(out.dst) + blockIdx.z * out.batch);
    const int n0 = tn * 64;
    const int k_lo = blockIdx.y * k_split, k_hi = min(K, k_lo + k_split);
    const int wm = (wv >> 1) * 32, wn = (wv & 1) * 32;
    f32x4 ra[2];
    u32x4 rb;
    const float *xp[2];
#pragma unroll
    for (int i = 0; i < 2; i++) {
        const int c = tid + 256 * i;
        int64_t r = min(m0 + (c >> 3), M - 1);
        if (src.rows) r = src.rows[r];
        xp[i] = reinterpret_cast<const float *>(src.x) + blockIdx.z * src.x_batch + r * src.ldx + (c & 7) * 4;
    }
    const uint16_t *wp = w + (int64_t)min(n0 + (tid >> 2), N - 1) * src.ldw + (tid & 3) * 8;
    auto fetch = [&](int k) {
        rb = *reinterpret_cast<const u32x4 *>(wp + k);
#pragma unroll
        for (int i = 0; i < 2; i++) ra[i] = *reinterpret_cast<const f32x4 *>(xp[i] + k);
    };
    auto stage = [&](int b) {
#pragma unroll
        for (int i = 0; i < 2; i++) {
            const int c = tid + 256 * i;
            *reinterpret_cast<f32x4 *>(&lds[b][(c >> 3) * DF_ROW + (c & 7) * 4]) = ra[i];
        }
        float *d = &lds[b][(64 + (tid >> 2)) * DF_ROW + (tid & 3) * 8];
        *reinterpret_cast<f32x4 *>(d) = f32x4{bf_lo(rb.x), bf_hi(rb.x), bf_lo(rb.y), bf_hi(rb.y)};
        *reinterpret_cast<f32x4 *>(d + 4) = f32x4{bf_lo(rb.z), bf_hi(rb.z), bf_lo(rb.w), bf_hi(rb.w)};
    };
    f32x4 acc[2][2];
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int j = 0; j < 2; j++) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    fetch(k_lo);
    stage(0);
    __syncthreads();
    int cur = 0;
    const int lr = lane & 15, lk = lane >> 4;
    for (int k = k_lo; k < k_hi; k += 32) {
        const bool more = k + 32 < k_hi;
        if (more) fetch(k + 32);
#pragma unroll
        for (int s = 0; s < 2; s++) {
            f32x4 fa[2], fb[2];
#pragma unroll
            for (int i = 0; i < 2; i++) {
                fa[i] = *reinterpret_cast<const f32x4 *>(&lds[cur][(wm + 16 * i + lr) * DF_ROW + 16 * s + 4 * lk]);
                fb[i] = *reinterpret_cast<const f32x4 *>(&lds[cur][(64 + wn + 16 * i + lr) * DF_ROW + 16 * s + 4 * lk]);
            }
#pragma unroll
            for (int e = 0; e < 4; e++)
#pragma unroll
                for (int i = 0; i < 2; i++)
#pragma unroll
                    for (int j = 0; j < 2; j++) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(fb[j][e], fa[i][e], acc[i][j], 0, 0, 0);
        }
        if (more) {
            stage(cur ^ 1);
            __syncthreads();
            cur ^= 1;
        }
    }
#pragma unroll
    for (int i = 0; i < 2; i++) {
        const int64_t m = m0 + wm + 16 * i + lr;
        if (m >= M) continue;
#pragma unroll
        for (int j = 0; j < 2; j++) {
            const int n = n0 + wn + 16 * j + 4 * lk;
            if (n < N) emit4(out, acc[i][j], m, n, M, N, blockIdx.y);
        }
    }
}

// the planes of a k split, added in order
__global__ __launch_bounds__(256) void dense_planes_kernel(Out out, int64_t M, int N, int splits) {
    const int64_t groups = out.n4 >> 2;
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= M * groups) return;
    const int64_t m = i / groups;
    const int n = (int)(i - m * groups) * 4;
    f32x4 v = *reinterpret_cast<const f32x4 *>(out.planes + m * out.n4 + n);
    for (int s = 1; s < splits; s++) v += *reinterpret_cast<const f32x4 *>(out.planes + ((int64_t)s * M + m) * out.n4 + n);
    Out o = out;
    o.planes = nullptr;
    emit4(o, v, m, n, M, N, 0);
}

struct Plan {
    int bm, bn, tiles_m, tiles_n, splits, k_split;
};

Plan plan(int precision, int64_t m, int64_t n, int64_t k) {
    Plan p;
    auto tiles = [&](int bm, int bn) { return ((m + bm - 1) / bm) * ((n + bn - 1) / bn); };
    if (precision == CQ_DENSE_F32) {
        p.bm = p.bn = 64;
    } else if (m > 64 && tiles(128, 128) * (k / 512) >= 256) {      // the large tile where splitting k can still fill the chip
        p.bm = p.bn = 128;
    } else if (m > 32) {
        p.bm = p.bn = 64;
    } else {
        p.bm = 32;
        p.bn = 64;
    }
    p.tiles_m = (int)((m + p.bm - 1) / p.bm);
    p.tiles_n = (int)((n + p.bn - 1) / p.bn);
    // enough workgroups for two per CU, each with at least 256 of k
    const int64_t t = (int64_t)p.tiles_m * p.tiles_n;
    int64_t s = t >= 384 ? 1 : (512 + t - 1) / t;
    s = s < k / 256 ? s : k / 256;
    s = s < 1 ? 1 : (s > 16 ? 16 : s);
    p.k_split = (int)((k / 64 + s - 1) / s) * 64;
    p.splits = (int)((k + p.k_split - 1) / p.k_split);
    return p;
}

// ---- one row --------------------------------------------------------------------------------------------------------------
// 8 waves; a wave takes one weight row at a time and walks it in blocks of 64 lanes x 8 elements x 4, one block ahead; the first
// block is requested before the prologue.  Weights are read once per step: non-temporal loads (33.3 -> 27.1 us on 4096 x 14336).  At most two
// workgroups per CU, which then walk the rows together.  The input row sits in LDS as f32, zero beyond `dim` and up to a whole block.
constexpr int MV_U = 4, MV_BLOCK = 512 * MV_U;
template <int PRO>
__global__ __launch_bounds__(512) void dense_matvec_kernel(const uint16_t *__restrict__ w, int64_t ldw, const float *__restrict__ x,
                                                           const float *__restrict__ vec, float eps, int dim, float *dst, const float *add, int accumulate,
                                                           int n, int k) {
    constexpr int U = MV_U, BLOCK = MV_BLOCK;
    extern __shared__ __attribute__((aligned(16))) float xs[];           // k rounded up to BLOCK
    __shared__ float red[8];
    const int tid = threadIdx.x, lane = tid & 63, wv = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int step = gridDim.x * 8, kb_n = (k + BLOCK - 1) / BLOCK;
    int r = blockIdx.x * 8 + wv;
    u32x4 cur[U], nxt[U];
    auto load = [&](int row, int kb, u32x4 (&d)[U]) {
        const uint16_t *p = w + (int64_t)row * ldw;
#pragma unroll
        for (int u = 0; u < U; u++) d[u] = __builtin_nontemporal_load(reinterpret_cast<const u32x4 *>(p + min(kb * BLOCK + u * 512 + lane * 8, k - 8)));
    };
    if (r < n) load(r, 0, cur);

    // the input row into LDS, several 16-byte loads per thread in flight (it comes from another kernel's hands, far away)
    constexpr int PF = PRO == CQ_DENSE_POLY || PRO == CQ_DENSE_RELU2 ? 8 : 4;
    const int n4 = kb_n * BLOCK / 4;
    f32x4 *xs4 = reinterpret_cast<f32x4 *>(xs);
    float s2 = 0.0f, s4 = 0.0f, s6 = 0.0f;
    for (int i0 = tid; i0 < n4; i0 += 512 * PF) {
        f32x4 v[PF];
#pragma unroll
        for (int j = 0; j < PF; j++) v[j] = *reinterpret_cast<const f32x4 *>(x + min(4 * (i0 + 512 * j), k - 4));
#pragma unroll
        for (int j = 0; j < PF; j++) {
            const int i = i0 + 512 * j;
            if (i >= n4) break;
#pragma unroll
            for (int e = 0; e < 4; e++) {
                const float z = 4 * i + e < dim ? v[j][e] : 0.0f, q = z * z;
                v[j][e] = PRO == CQ_DENSE_RELU2 ? (z > 0.0f ? q : 0.0f) : z;
                if (PRO == CQ_DENSE_LAYER_NORM) s2 += z;
                else if (PRO != CQ_DENSE_PLAIN) s2 += q;
                if (PRO == CQ_DENSE_POLY) {
                    s4 = fmaf(q, q, s4);
                    s6 = fmaf(q * q, q, s6);
                }
            }
            xs4[i] = v[j];
        }
    }
    if (PRO == CQ_DENSE_NORM) {
        const float m = sqrtf(block_sum_512(s2, red) / (float)dim + eps);
        for (int i = tid; i < dim; i += 512) xs[i] = xs[i] / m * vec[i];
    } else if (PRO == CQ_DENSE_LAYER_NORM) {
        layer_norm_lds_512(xs, dim, s2, vec, eps, red);
    } else if (PRO == CQ_DENSE_POLY) {
        const float inv = 1.0f / (float)dim;
        const float i1 = vec[0] / sqrtf(block_sum_512(s2, red) * inv + eps);
        const float i2 = vec[1] / sqrtf(block_sum_512(s4, red) * inv + eps);
        const float i3 = vec[2] / sqrtf(block_sum_512(s6, red) * inv + eps);
        const float e = vec[3];
        for (int i = tid; i < n4; i += 512) {
            f32x4 v = xs4[i];
#pragma unroll
            for (int j = 0; j < 4; j++) {
                const float q = v[j] * v[j];
                v[j] = 4 * i + j < dim ? fmaf(i1, v[j], fmaf(i2, q, fmaf(i3, q * v[j], e))) : 0.0f;
            }
            xs4[i] = v;
        }
    }
    __syncthreads();

    for (; r < n; r += step) {
        float acc[2] = {0.0f, 0.0f};
        for (int kb = 0; kb < kb_n; kb++) {
            const bool last = kb + 1 == kb_n;
            const int next = last ? r + step : r;
            if (next < n) load(next, last ? 0 : kb + 1, nxt);
#pragma unroll
            for (int u = 0; u < U; u++) {
                const f32x4 *xv = reinterpret_cast<const f32x4 *>(xs + kb * BLOCK + u * 512 + lane * 8);
                const f32x4 a = xv[0], b = xv[1];
                dot8(cur[u], a, b, acc);
            }
#pragma unroll
            for (int u = 0; u < U; u++) cur[u] = nxt[u];
        }
        const float s = wave_sum(acc[0] + acc[1]);
        if (lane == 0) dst[r] = s + (accumulate ? dst[r] : 0.0f) + (add ? add[r] : 0.0f);
    }
}

template <int PRO>
int matvec_launch(const uint16_t *w, int64_t ldw, const float *x, const float *vec, float eps, int dim, float *dst, const float *add, int accumulate, int n,
                  int k, hipStream_t s) {
    const size_t lds = (size_t)((k + MV_BLOCK - 1) / MV_BLOCK) * MV_BLOCK * sizeof(float);
    const int blocks = (n + 7) / 8 < 512 ? (n + 7) / 8 : 512;
    if (lds > 64 * 1024) {
        const int e = (int)hipFuncSetAttribute(reinterpret_cast<const void *>(dense_matvec_kernel<PRO>), hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024 - 64);
        if (e) return e;
    }
    hipLaunchKernelGGL(dense_matvec_kernel<PRO>, dim3(blocks), dim3(512), lds, s, w, ldw, x, vec, eps, dim, dst, add, accumulate, n, k);
    return (int)hipGetLastError();
}

}  // namespace

extern "C" {

int64_t cq_dense_matmul_workspace_bytes(int precision, int64_t m, int64_t n, int64_t k) {
    if (m <= 0 || n <= 0 || k <= 0 || k % 64) return 0;
    const Plan p = plan(precision, m, n, k);
    return p.splits > 1 ? (int64_t)p.splits * m * ((n + 3) / 4 * 4) * 4 : 0;
}

int cq_dense_product(int precision, const cq_dense_args *args, void *workspace_dev, int64_t workspace_bytes, void *stream) {
    if (!args) return CQ_ERR_NULL;
    const cq_dense_args &a = *args;
    if (precision != CQ_DENSE_BF16 && precision != CQ_DENSE_F32) return CQ_ERR_DTYPE;
    if (precision == CQ_DENSE_F32 && (a.x_bf16 || a.dst_bf16)) return CQ_ERR_DTYPE;
    if (a.act < CQ_DENSE_ACT_NONE || a.act > CQ_DENSE_ACT_SWIGLU) return CQ_ERR_DTYPE;
    const int64_t m = a.m, n = a.n, k = a.k, cols = a.act == CQ_DENSE_ACT_SWIGLU ? n / 2 : n;
    if (m < 0 || n < 0 || k <= 0 || k % 64 || a.ldw % 64 || a.ldw < k || a.ldx % (a.x_bf16 ? 8 : 4) || a.ldx < k || a.ldd < cols || (a.add_dev && a.ld_add < cols) ||
        a.batch < 1)
        return CQ_ERR_SHAPE;
    if ((a.act == CQ_DENSE_ACT_SWIGLU && n % 2) || ((a.act || a.dst_bf16) && (a.accumulate || a.add_dev))) return CQ_ERR_SHAPE;
    if (a.batch > 1 && (a.accumulate || a.add_dev || a.row_scale_dev || a.tiles_dev || a.w_batch % 8 || a.x_batch % (a.x_bf16 ? 8 : 4))) return CQ_ERR_SHAPE;
    if (a.tiles_dev && (a.max_tiles < 1 || a.accumulate || a.add_dev || a.w_batch % 8 || (a.tile_rows != 32 && a.tile_rows != 64 && a.tile_rows != 128) ||
                        (precision == CQ_DENSE_F32 && a.tile_rows != 64)))
        return CQ_ERR_SHAPE;
    if (m == 0 || n == 0) return CQ_OK;
    if (!a.w_dev || !a.x_dev || !a.dst_dev || (a.tiles_dev && !a.n_tiles_dev)) return CQ_ERR_NULL;
    if (misaligned(a.w_dev, 16) || misaligned(a.x_dev, 16) || misaligned(a.dst_dev, a.dst_bf16 ? 2 : 4) || misaligned(a.add_dev, 4) || misaligned(workspace_dev, 16) ||
        misaligned(a.row_scale_dev, 4))
        return CQ_ERR_ALIGN;
    if (m > (1 << 24) || n > (1 << 24) || k > (1 << 24) || a.batch > 65535) return CQ_ERR_RANGE;
    Plan p = plan(precision, m, n, k);
    if (a.batch > 1 || a.tiles_dev) {
        if (a.tiles_dev) {
            p.bm = (int)a.tile_rows;
            p.bn = p.bm == 128 ? 128 : 64;
            p.tiles_m = (int)a.max_tiles;
        }
        p.tiles_n = (int)((n + p.bn - 1) / p.bn);
        p.splits = 1;
        p.k_split = (int)k;
    }
    if ((int64_t)p.tiles_m * p.tiles_n > 0x7fffffffLL) return CQ_ERR_RANGE;
    if (p.splits > 1 && (!workspace_dev || workspace_bytes < cq_dense_matmul_workspace_bytes(precision, m, n, k))) return CQ_ERR_WORKSPACE;
    Out o;
    o.dst = a.dst_dev;
    o.add = a.add_dev;
    o.ldd = a.ldd;
    o.ld_add = a.ld_add;
    o.accumulate = a.accumulate;
    o.planes = p.splits > 1 ? (float *)workspace_dev : nullptr;
    o.n4 = (n + 3) / 4 * 4;
    o.act = a.act;
    o.bf16 = a.dst_bf16;
    o.row_scale = a.row_scale_dev;
    o.rows = a.dst_rows_dev;
    o.batch = a.batch > 1 ? a.dst_batch : 0;
    Src src;
    src.w = (const uint16_t *)a.w_dev;
    src.x = a.x_dev;
    src.ldw = a.ldw;
    src.ldx = a.ldx;
    src.w_batch = a.w_batch;
    src.x_batch = a.x_batch;
    src.rows = a.src_rows_dev;
    src.tiles = a.tiles_dev;
    src.n_tiles = a.n_tiles_dev;
    hipStream_t s = (hipStream_t)stream;
    const dim3 grid((unsigned)(p.tiles_m * p.tiles_n), (unsigned)p.splits, (unsigned)a.batch);
#define CQ_DM(K_) hipLaunchKernelGGL(K_, grid, dim3(256), 0, s, src, o, m, (int)n, (int)k, p.tiles_m, p.tiles_n, p.k_split)
    if (precision == CQ_DENSE_F32) CQ_DM(dense_f32_kernel);
    else if (p.bm == 128 && a.x_bf16) CQ_DM((dense_bf16_kernel<128, 128, 2, 2, true>));
    else if (p.bm == 128) CQ_DM((dense_bf16_kernel<128, 128, 2, 2, false>));
    else if (p.bm == 64 && a.x_bf16) CQ_DM((dense_bf16_kernel<64, 64, 2, 2, true>));
    else if (p.bm == 64) CQ_DM((dense_bf16_kernel<64, 64, 2, 2, false>));
    else if (a.x_bf16) CQ_DM((dense_bf16_kernel<32, 64, 1, 4, true>));
    else CQ_DM((dense_bf16_kernel<32, 64, 1, 4, false>));
#undef CQ_DM
    if (p.splits > 1)
        hipLaunchKernelGGL(dense_planes_kernel, dim3((unsigned)((m * (o.n4 / 4) + 255) / 256)), dim3(256), 0, s, o, m, (int)n, p.splits);
    return (int)hipGetLastError();
}

int cq_dense_matmul(int precision, const void *w_dev, int64_t ldw, const float *x_dev, int64_t ldx, float *dst_dev, int64_t ldd, const float *add_dev,
                    int64_t ld_add, int accumulate, int64_t m, int64_t n, int64_t k, void *workspace_dev, int64_t workspace_bytes, void *stream) {
    cq_dense_args a = {};
    a.w_dev = w_dev;
    a.ldw = ldw;
    a.x_dev = x_dev;
    a.ldx = ldx;
    a.dst_dev = dst_dev;
    a.ldd = ldd;
    a.add_dev = add_dev;
    a.ld_add = ld_add;
    a.accumulate = accumulate;
    a.m = m;
    a.n = n;
    a.k = k;
    a.batch = 1;
    return cq_dense_product(precision, &a, workspace_dev, workspace_bytes, stream);
}

int cq_dense_matvec(const void *w_dev, int64_t ldw, const float *x_dev, int prologue, const float *vec_dev, float eps, int64_t dim, float *dst_dev,
                    const float *add_dev, int accumulate, int64_t n, int64_t k, void *stream) {
    if (n < 0 || k <= 0 || k % 64 || ldw % 64 || ldw < k || dim <= 0 || dim > k) return CQ_ERR_SHAPE;
    if (prologue < CQ_DENSE_PLAIN || prologue > CQ_DENSE_RELU2) return CQ_ERR_DTYPE;
    if (n == 0) return CQ_OK;
    if (!w_dev || !x_dev || !dst_dev || (prologue != CQ_DENSE_PLAIN && prologue != CQ_DENSE_RELU2 && !vec_dev)) return CQ_ERR_NULL;
    if (misaligned(w_dev, 16) || misaligned(x_dev, 16) || misaligned(vec_dev, 4) || misaligned(dst_dev, 4) || misaligned(add_dev, 4)) return CQ_ERR_ALIGN;
    if (k > CQ_DENSE_MATVEC_MAX_K || n > (1 << 24)) return CQ_ERR_RANGE;
    const uint16_t *w = (const uint16_t *)w_dev;
    hipStream_t s = (hipStream_t)stream;
#define CQ_MV(P_) case P_: return matvec_launch<P_>(w, ldw, x_dev, vec_dev, eps, (int)dim, dst_dev, add_dev, accumulate, (int)n, (int)k, s)
    switch (prologue) {
        CQ_MV(CQ_DENSE_NORM);
        CQ_MV(CQ_DENSE_POLY);
        CQ_MV(CQ_DENSE_LAYER_NORM);
        CQ_MV(CQ_DENSE_RELU2);
        default: return matvec_launch<CQ_DENSE_PLAIN>(w, ldw, x_dev, vec_dev, eps, (int)dim, dst_dev, add_dev, accumulate, (int)n, (int)k, s);
    }
#undef CQ_MV
}

}  // extern "C"
