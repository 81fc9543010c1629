// Attention over latents: what a position leaves in the cache is one row shared by all heads, a normed latent c and a rotated key part.
// A head's unrotated key is W_uk c and its value W_uv c.  Two ways to the same result:
//   expanded   keys and values of all heads are computed (a dense product over the cache rows) and attended to head by head: many query rows
//   absorbed   W_uk is applied to the query instead and W_uv to the attended latent: every head attends to the cache rows themselves, few query rows
// T is the type that the products read: bfloat16, or float for products in f32.  Scores, weights and sums are f32.  Queries are packed with the scale and
// log2(e) multiplied in, so that a weight is a power of two.
#include "cq_dense.h"
#include "cq_mix.h"

namespace {

// ---- operands in 16-byte chunks: four chunks side by side (one per lane group) are one step of a product ------------------------------
template <typename T> struct Chunk {
    static constexpr int N = 16 / sizeof(T);               // elements
    static constexpr int STEP = 4 * N;
    static constexpr int KEYS = 128 / sizeof(T);           // keys per tile: a row of transposed values is eight chunks
};
template <typename T> __device__ __forceinline__ f32x4 mma(const u32x4 &a, const u32x4 &b, f32x4 c);
template <> __device__ __forceinline__ f32x4 mma<__bf16>(const u32x4 &a, const u32x4 &b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}
template <> __device__ __forceinline__ f32x4 mma<float>(const u32x4 &a, const u32x4 &b, f32x4 c) {
    const f32x4 x = __builtin_bit_cast(f32x4, a), y = __builtin_bit_cast(f32x4, b);
#pragma unroll
    for (int e = 0; e < 4; e++) c = mfma4(x[e], y[e], c);
    return c;
}

// Weights are taken relative to a reference that follows the running maximum only when that is more than this far ahead (in powers of two): sums and outputs
// are rarely rescaled, and no weight exceeds 2^8.
constexpr float LAG = 8.0f;

// LDS chunk of 16 bytes `c` of key row r (rows of a multiple of eight chunks) and of value column r (eight chunks of keys)
__device__ __forceinline__ int key_slot(int r, int c) { return c ^ (r & 7); }
__device__ __forceinline__ int value_slot(int r, int c) { return c ^ ((r ^ (r >> 3)) & 7); }

// In columns of every other block of 64 the two halves of a bf16 chunk change places, so that the lanes of a store fall on all banks; so do the weights for them.
// Values of keys 4 a .. 4 a + 3, columns of chunk cg, transposed into LDS: [column][key].  The keys of a row are ordered so that the chunk that a lane reads
// holds the keys whose scores it has: for bf16 4 lk .. 4 lk + 3 of two neighbouring tiles of 16.
template <typename T> __device__ __forceinline__ void store_values(u32x4 *vs, int a, int cg, const u32x4 (&v)[4]);
template <> __device__ __forceinline__ void store_values<__bf16>(u32x4 *vs, int a, int cg, const u32x4 (&v)[4]) {
    const int chunk = (a >> 3) * 4 + (a & 3), half = ((a >> 2) ^ (cg >> 3)) & 1;
#pragma unroll
    for (int j = 0; j < 8; j++) {
        const int r = cg * 8 + j, w = j >> 1;
        const uint32_t pick = j & 1 ? 0x07060302u : 0x05040100u;           // the high or low halves of two registers
        u32x2 x;
        x.x = __builtin_amdgcn_perm(v[1][w], v[0][w], pick);
        x.y = __builtin_amdgcn_perm(v[3][w], v[2][w], pick);
        reinterpret_cast<u32x2 *>(vs + r * 8 + value_slot(r, chunk))[half] = x;
    }
}
template <> __device__ __forceinline__ void store_values<float>(u32x4 *vs, int a, int cg, const u32x4 (&v)[4]) {
#pragma unroll
    for (int j = 0; j < 4; j++) {
        const int r = cg * 4 + j;
        vs[r * 8 + value_slot(r, a)] = u32x4{v[0][j], v[1][j], v[2][j], v[3][j]};
    }
}

// weights of a lane's keys (tiles of 16 in order, four keys each) as operand chunk s
template <typename T> __device__ __forceinline__ u32x4 weight_chunk(const f32x4 *p, int s);
template <> __device__ __forceinline__ u32x4 weight_chunk<__bf16>(const f32x4 *p, int s) {
    bf16x8 r;
#pragma unroll
    for (int i = 0; i < 4; i++) {
        r[i] = (__bf16)p[2 * s][i];
        r[4 + i] = (__bf16)p[2 * s + 1][i];
    }
    return __builtin_bit_cast(u32x4, r);
}
template <> __device__ __forceinline__ u32x4 weight_chunk<float>(const f32x4 *p, int s) { return __builtin_bit_cast(u32x4, p[s]); }
// ... for the columns of block b of 64
template <typename T> __device__ __forceinline__ u32x4 for_block(const u32x4 &w, int b) { return sizeof(T) == 2 && (b & 1) ? u32x4{w.z, w.w, w.x, w.y} : w; }

// over the four lanes that share lane & 15
__device__ __forceinline__ float group_max(float v) {
    v = fmaxf(v, __shfl_xor(v, 16, 64));
    return fmaxf(v, __shfl_xor(v, 32, 64));
}
__device__ __forceinline__ float group_sum(float v) {
    v += __shfl_xor(v, 16, 64);
    return v + __shfl_xor(v, 32, 64);
}

// ---- expanded: causal attention head by head ---------------------------------------------------------------------------------------------
// Workgroup: four waves of 16 NQ query rows of one head; tiles of keys through LDS, the next one on its way in registers.  Scores come out
// transposed (key x query), so a lane holds one query's keys and its weights are the operand of the value product as they are; the outputs
// come out as value column x query.
struct Expanded {
    const void *q, *k, *kr, *v;                            // [row][head], [key][head], [key], [key][head]
    int64_t q_row, k_row, kr_row, v_row;
    int q_head, k_head, v_head, d1, d2, vdim, v_pad;       // d1: unrotated dimensions (padded), d2: rotated
    const float *gate;
    int64_t gate_row;
    void *out;                                             // of type T, like everything that only feeds a product
    int64_t out_row;
    int pos, rows, heads;
};

template <typename T, int DK, int DV, int NQ>
__global__ __launch_bounds__(256) void latent_expanded_kernel(Expanded p) {
    constexpr int CH = Chunk<T>::N, KT = Chunk<T>::KEYS, NT = KT / 16, NKF = DK / Chunk<T>::STEP, KC = DK / CH, NVF = DV / 16, BM = 64 * NQ;
    constexpr int KL = KT * KC / 256, VT = (KT / 4) * (DV / CH), VL = (VT + 255) / 256;
    __shared__ u32x4 ks[KT * KC], vs[DV * 8];
    const int tid = threadIdx.x, lane = tid & 63, wv = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lk = lane >> 4;
    // The longest rows first; where two workgroups per CU hold them all, the shortest join the longest.  With heads in eighths a head stays on one XCD, whose L2
    // then holds its keys and values.
    const int blocks = (p.rows + BM - 1) / BM, per = p.heads >> 3, total = blocks * p.heads;
    const bool split = (p.heads & 7) == 0;
    const int n = split ? total >> 3 : total, half = (n + 1) / 2, turn = split ? blockIdx.x >> 3 : blockIdx.x;
    const int rank = NQ == 1 && total <= 512 && turn >= half ? n - 1 - (turn - half) : turn, heads = split ? per : p.heads;
    const int h = (split ? (blockIdx.x & 7) * per : 0) + rank % heads, block = blocks - 1 - rank / heads;
    const int m0 = block * BM, mw = m0 + wv * 16 * NQ;
    const int last = p.pos + min(m0 + BM, p.rows) - 1, n_tiles = last / KT + 1, dk = p.d1 + p.d2;
    const T *kb = (const T *)p.k + (int64_t)h * p.k_head, *krb = (const T *)p.kr, *vb = (const T *)p.v + (int64_t)h * p.v_head;

    u32x4 qf[NQ][NKF];
    int pq[NQ];
#pragma unroll
    for (int i = 0; i < NQ; i++) {
        const int r = min(mw + 16 * i + lr, p.rows - 1);
        pq[i] = p.pos + r;
        const T *qr = (const T *)p.q + r * p.q_row + (int64_t)h * p.q_head;
#pragma unroll
        for (int s = 0; s < NKF; s++) {
            const int c = (4 * s + lk) * CH;
            qf[i][s] = c < dk ? *reinterpret_cast<const u32x4 *>(qr + c) : u32x4{0, 0, 0, 0};
        }
    }
    // where a thread's pieces of a tile come from: key row of the tile, address of the column, bytes from key to key.  Columns beyond the head meet zeros of
    // the query: any finite values will do.
    u32x4 rk[KL], rv[VL][4];
    const char *k_at[KL], *v_at[VL];
    uint32_t k_step[KL];
    const uint32_t v_step = (uint32_t)p.v_row * sizeof(T);
#pragma unroll
    for (int i = 0; i < KL; i++) {
        const int c = ((tid + 256 * i) % KC) * CH;
        const bool rotated = c >= p.d1 && c < dk;
        k_at[i] = (const char *)(rotated ? krb + (c - p.d1) : kb + (c < p.d1 ? c : 0));
        k_step[i] = (uint32_t)(rotated ? p.kr_row : p.k_row) * sizeof(T);
    }
#pragma unroll
    for (int i = 0; i < VL; i++) v_at[i] = (const char *)(vb + min((tid + 256 * i) / (KT / 4) * CH, p.v_pad - CH));
    auto fetch = [&](int j0) {
#pragma unroll
        for (int i = 0; i < KL; i++) rk[i] = *reinterpret_cast<const u32x4 *>(k_at[i] + (uint64_t)(uint32_t)min(j0 + (tid + 256 * i) / KC, last) * k_step[i]);
#pragma unroll
        for (int i = 0; i < VL; i++)
#pragma unroll
            for (int j = 0; j < 4; j++)
                rv[i][j] = *reinterpret_cast<const u32x4 *>(v_at[i] + (uint64_t)(uint32_t)min(j0 + 4 * ((tid + 256 * i) % (KT / 4)) + j, last) * v_step);
    };
    auto stage = [&]() {
#pragma unroll
        for (int i = 0; i < KL; i++) {
            const int idx = tid + 256 * i, r = idx / KC;
            ks[r * KC + key_slot(r, idx % KC)] = rk[i];
        }
#pragma unroll
        for (int i = 0; i < VL; i++) {
            const int idx = tid + 256 * i, a = idx % (KT / 4), cg = idx / (KT / 4);
            if (cg * CH < p.v_pad) store_values<T>(vs, a, cg, rv[i]);
        }
    };

    f32x4 o[NQ][NVF];
    float m_run[NQ], l_run[NQ];
#pragma unroll
    for (int i = 0; i < NQ; i++) {
        m_run[i] = -INFINITY;
        l_run[i] = 0.0f;
#pragma unroll
        for (int n = 0; n < NVF; n++) o[i][n] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    // LDS slots of a lane: key chunks 4 k + lk of row lr by parity of k, value chunks 4 sp + lk of column lr by (n & 3) ^ 2 sp
    const int ka[2] = {lr * KC + (lk ^ (lr & 7)), lr * KC + ((4 + lk) ^ (lr & 7))}, vx = lk ^ (lr & 7) ^ (lr >> 3);
    const int va[4] = {lr * 8 + vx, lr * 8 + (vx ^ 2), lr * 8 + (vx ^ 4), lr * 8 + (vx ^ 6)};
    fetch(0);
    for (int it = 0; it < n_tiles; it++) {
        const int j0 = it * KT;
        __syncthreads();
        stage();
        __syncthreads();
        if (it + 1 < n_tiles) fetch(j0 + KT);
        if (j0 > p.pos + mw + 16 * NQ - 1) continue;       // wave-uniform: nothing visible to this wave's rows
        f32x4 s[NQ][NT];
#pragma unroll
        for (int i = 0; i < NQ; i++)
#pragma unroll
            for (int t = 0; t < NT; t++) s[i][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < NKF; k++)
#pragma unroll
            for (int t = 0; t < NT; t++) {
                const u32x4 a = ks[ka[k & 1] + 8 * (k >> 1) + 16 * t * KC];
#pragma unroll
                for (int i = 0; i < NQ; i++) s[i][t] = mma<T>(a, qf[i][k], s[i][t]);
            }
        if (j0 + KT - 1 > p.pos + mw) {                    // some key of the tile lies after some row
#pragma unroll
            for (int i = 0; i < NQ; i++)
#pragma unroll
                for (int t = 0; t < NT; t++)
#pragma unroll
                    for (int e = 0; e < 4; e++) s[i][t][e] = j0 + 16 * t + 4 * lk + e > pq[i] ? -INFINITY : s[i][t][e];
        }
#pragma unroll
        for (int i = 0; i < NQ; i++) {
            float mx = s[i][0][0];
#pragma unroll
            for (int t = 0; t < NT; t++)
#pragma unroll
                for (int e = 0; e < 4; e++) mx = fmaxf(mx, s[i][t][e]);
            if (__any(mx > m_run[i] + LAG)) {              // in the first tile for every row: it sees key 0
                const float m = fmaxf(m_run[i], group_max(mx)), al = __builtin_amdgcn_exp2f(m_run[i] - m);
#pragma unroll
                for (int n = 0; n < NVF; n++) o[i][n] *= al;
                l_run[i] *= al;
                m_run[i] = m;
            }
            float sum[2] = {0.0f, 0.0f};
#pragma unroll
            for (int t = 0; t < NT; t++)
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    s[i][t][e] = __builtin_amdgcn_exp2f(s[i][t][e] - m_run[i]);
                    sum[e & 1] += s[i][t][e];
                }
            l_run[i] += sum[0] + sum[1];
        }
#pragma unroll
        for (int sp = 0; sp < 2; sp++) {
            u32x4 w[NQ];
#pragma unroll
            for (int i = 0; i < NQ; i++) w[i] = weight_chunk<T>(s[i], sp);
#pragma unroll
            for (int n = 0; n < NVF; n++) {
                const u32x4 a = vs[va[(n & 3) ^ (2 * sp)] + 128 * n];
#pragma unroll
                for (int i = 0; i < NQ; i++) o[i][n] = mma<T>(a, for_block<T>(w[i], n >> 2), o[i][n]);
            }
        }
    }
    const bool vec = p.vdim % 4 == 0 && p.out_row % 4 == 0;
#pragma unroll
    for (int i = 0; i < NQ; i++) {
        const int r = mw + 16 * i + lr;
        const float l = group_sum(l_run[i]);
        if (r >= p.rows) continue;
        const float f = mix_sigmoid(p.gate[r * p.gate_row + h]) / l;
        T *dst = (T *)p.out + r * p.out_row + (int64_t)h * p.vdim;
#pragma unroll
        for (int n = 0; n < NVF; n++) {
            const int c = 16 * n + 4 * lk;
            if (vec) {
                if (c < p.vdim) {
                    typedef T T4 __attribute__((ext_vector_type(4)));
                    T4 v;
#pragma unroll
                    for (int e = 0; e < 4; e++) v[e] = (T)(o[i][n][e] * f);
                    *reinterpret_cast<T4 *>(dst + c) = v;
                }
            } else {
#pragma unroll
                for (int e = 0; e < 4; e++)
                    if (c + e < p.vdim) dst[c + e] = (T)(o[i][n][e] * f);
            }
        }
    }
}

// ---- absorbed: every (row, head) attends to the cache rows themselves ------------------------------------------------------------------------
// Workgroup: 16 NQ of the rows * heads queries, all on the same keys.  Per tile: a wave takes half of the keys and half of the columns of the scores (a quarter of
// the query registers), every wave does the softmax of all queries from the sums in LDS, and takes every fourth 16 columns of the latent in the value
// product.  A cache row is read once for both products.
// blockIdx.z: split of the key tiles.
struct Absorbed {
    const void *q, *cache;                                 // [row][head][ld], [key][ld]: rank_pad latent columns, then the rotated part
    int ld, rank_pad, heads, rows, pos, ctx;
    const int32_t *pos_dev;
    const float *gate;
    int64_t gate_row;
    float *out;                                            // [row][head][rank_pad], gated
    float *part;                                           // records instead: [split][query][rank_pad] unnormalized, then [split][query] of (maximum, sum)
};

// A key row in LDS: DV latent columns, then DR rotated ones, zero where the cache row has none.
template <typename T, int DV, int DR, int NQ>
__global__ __launch_bounds__(256, 1) void latent_absorbed_kernel(Absorbed p) {
    constexpr int CH = Chunk<T>::N, KT = Chunk<T>::KEYS, NT = KT / 16, NKF = (DV + DR) / Chunk<T>::STEP, KC = (DV + DR) / CH, NVW = DV / 64, BM = 16 * NQ, SS = KT + 4;
    // a thread's pieces: four keys x one chunk, latent ones (AL groups of keys apart) and rotated ones
    constexpr int NC = DV / CH, AL = 256 / NC, TL = KT / 4 / AL, NR = DR / CH, RT = (KT / 4) * NR, RL = (RT + 255) / 256;
    constexpr int NKH = NKF / 2, NTH = NT / 2;             // steps and tiles of keys of a wave's scores
    static_assert(256 % NC == 0 && (KT / 4) % AL == 0 && NKF % 2 == 0, "pieces");
    extern __shared__ __attribute__((aligned(16))) u32x4 lds[];
    u32x4 *ks = lds, *vs = ks + KT * KC;
    float *ss = reinterpret_cast<float *>(vs + DV * 8);    // scores [half of the columns][query][key]
    const int tid = threadIdx.x, lane = tid & 63, wv = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lk = lane >> 4;
    const int M = p.rows * p.heads, m0 = blockIdx.x * BM, nz = gridDim.z, z = blockIdx.z;
    const int pos = p.pos + (p.pos_dev ? p.pos_dev[0] : 0);
    if (pos + p.rows > p.ctx) return;
    const int last = pos + (min(m0 + BM, M) - 1) / p.heads, n_tiles = last / KT + 1;
    const int lo = (int)((uint32_t)n_tiles * z / (uint32_t)nz), hi = (int)((uint32_t)n_tiles * (z + 1) / (uint32_t)nz);
    const T *cache = (const T *)p.cache;

    // cache pieces first, then the queries (where the cache row has no column, the query's value does not matter)
    u32x4 rg[TL][4], rr[RL][4];
    const int ca = (tid % NC) * CH, a0 = tid / NC;
    auto fetch = [&](int j0) {
#pragma unroll
        for (int i = 0; i < TL; i++)
#pragma unroll
            for (int j = 0; j < 4; j++) {
                rg[i][j] = u32x4{0, 0, 0, 0};
                if (ca < p.rank_pad) rg[i][j] = *reinterpret_cast<const u32x4 *>(cache + (int64_t)min(j0 + 4 * (a0 + AL * i) + j, last) * p.ld + ca);
            }
#pragma unroll
        for (int i = 0; i < RL; i++) {
            const int idx = tid + 256 * i, a = idx / NR, c = (idx % NR) * CH;
#pragma unroll
            for (int j = 0; j < 4; j++) {
                rr[i][j] = u32x4{0, 0, 0, 0};
                if (c < p.ld - p.rank_pad && idx < RT) rr[i][j] = *reinterpret_cast<const u32x4 *>(cache + (int64_t)min(j0 + 4 * a + j, last) * p.ld + p.rank_pad + c);
            }
        }
    };
    auto stage = [&]() {
#pragma unroll
        for (int i = 0; i < TL; i++) {
            const int a = a0 + AL * i, c = tid % NC;
#pragma unroll
            for (int j = 0; j < 4; j++) ks[(4 * a + j) * KC + key_slot(4 * a + j, c)] = rg[i][j];
            store_values<T>(vs, a, c, rg[i]);
        }
#pragma unroll
        for (int i = 0; i < RL; i++) {
            const int idx = tid + 256 * i, a = idx / NR, c = NC + idx % NR;
            if (idx < RT)
#pragma unroll
                for (int j = 0; j < 4; j++) ks[(4 * a + j) * KC + key_slot(4 * a + j, c)] = rr[i][j];
        }
    };
    if (lo < hi) fetch(lo * KT);
    const int k0 = (wv & 1) * NKH, t0 = (wv >> 1) * NTH;
    u32x4 qf[NQ][NKH];
#pragma unroll
    for (int i = 0; i < NQ; i++) {
        const T *qr = (const T *)p.q + (int64_t)min(m0 + 16 * i + lr, M - 1) * p.ld;
#pragma unroll
        for (int s = 0; s < NKH; s++) {
            const int k = k0 + s, c = (4 * k + lk) * CH;   // a step lies in one of the two parts
            qf[i][s] = *reinterpret_cast<const u32x4 *>(qr + min(4 * k < NC ? min(c, p.rank_pad - CH) : p.rank_pad + c - DV, p.ld - CH));
        }
    }
    int pq[NQ];
#pragma unroll
    for (int i = 0; i < NQ; i++) pq[i] = pos + min(m0 + 16 * i + lr, M - 1) / p.heads;

    f32x4 o[NQ][NVW];
    float m_run[NQ], l_run[NQ];
#pragma unroll
    for (int i = 0; i < NQ; i++) {
        m_run[i] = -INFINITY;
        l_run[i] = 0.0f;
#pragma unroll
        for (int n = 0; n < NVW; n++) o[i][n] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    for (int it = lo; it < hi; it++) {
        const int j0 = it * KT;
        __syncthreads();
        stage();
        __syncthreads();
        if (it + 1 < hi) fetch(j0 + KT);
        {
            f32x4 s[NQ][NTH];
#pragma unroll
            for (int i = 0; i < NQ; i++)
#pragma unroll
                for (int t = 0; t < NTH; t++) s[i][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k = 0; k < NKH; k++)
#pragma unroll
                for (int t = 0; t < NTH; t++) {
                    const u32x4 a = ks[(16 * (t0 + t) + lr) * KC + key_slot(lr, 4 * (k0 + k) + lk)];
#pragma unroll
                    for (int i = 0; i < NQ; i++) s[i][t] = mma<T>(a, qf[i][k], s[i][t]);
                }
#pragma unroll
            for (int i = 0; i < NQ; i++)
#pragma unroll
                for (int t = 0; t < NTH; t++) *reinterpret_cast<f32x4 *>(ss + ((wv & 1) * BM + 16 * i + lr) * SS + 16 * (t0 + t) + 4 * lk) = s[i][t];
        }
        __syncthreads();
        u32x4 w[NQ][2];
#pragma unroll
        for (int i = 0; i < NQ; i++) {
            f32x4 s[NT];
            float mx = -INFINITY, sum = 0.0f;
#pragma unroll
            for (int t = 0; t < NT; t++) {
                const float *sum_of = ss + (16 * i + lr) * SS + 16 * t + 4 * lk;
                s[t] = *reinterpret_cast<const f32x4 *>(sum_of) + *reinterpret_cast<const f32x4 *>(sum_of + BM * SS);
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    s[t][e] = j0 + 16 * t + 4 * lk + e > pq[i] ? -INFINITY : s[t][e];
                    mx = fmaxf(mx, s[t][e]);
                }
            }
            if (__any(mx > m_run[i] + LAG)) {
                const float m = fmaxf(m_run[i], group_max(mx)), al = m > -INFINITY ? __builtin_amdgcn_exp2f(m_run[i] - m) : 1.0f;
#pragma unroll
                for (int n = 0; n < NVW; n++) o[i][n] *= al;
                l_run[i] *= al;
                m_run[i] = m;
            }
            const float base = m_run[i] > -INFINITY ? m_run[i] : 0.0f;                 // a row before all keys of the split: weights of zero
#pragma unroll
            for (int t = 0; t < NT; t++)
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    s[t][e] = __builtin_amdgcn_exp2f(s[t][e] - base);
                    sum += s[t][e];
                }
            l_run[i] += sum;
#pragma unroll
            for (int sp = 0; sp < 2; sp++) w[i][sp] = weight_chunk<T>(s, sp);
        }
#pragma unroll
        for (int n = 0; n < NVW; n++) {                    // columns beyond the latent are zero
            const int r = 64 * n + 16 * wv + lr;
#pragma unroll
            for (int sp = 0; sp < 2; sp++) {
                const u32x4 a = vs[r * 8 + value_slot(r, 4 * sp + lk)];
#pragma unroll
                for (int i = 0; i < NQ; i++) o[i][n] = mma<T>(a, for_block<T>(w[i][sp], n), o[i][n]);
            }
        }
    }
#pragma unroll
    for (int i = 0; i < NQ; i++) {
        const int m = m0 + 16 * i + lr;
        const float l = group_sum(l_run[i]);
        if (m >= M) continue;
        float f = 1.0f;
        float *dst;
        if (p.part) {
            dst = p.part + ((int64_t)z * M + m) * p.rank_pad;
            if (wv == 0 && lk == 0) {
                float *ml = p.part + (int64_t)nz * M * p.rank_pad + 2 * ((int64_t)z * M + m);
                ml[0] = m_run[i];
                ml[1] = l;
            }
            if (lo >= hi) continue;                        // nothing but the (empty) sum
        } else {
            dst = p.out + (int64_t)m * p.rank_pad;
            f = mix_sigmoid(p.gate[(m / p.heads) * p.gate_row + m % p.heads]) / l;
        }
#pragma unroll
        for (int n = 0; n < NVW; n++) {
            const int c = 64 * n + 16 * wv + 4 * lk;
            if (c < p.rank_pad) *reinterpret_cast<f32x4 *>(dst + c) = o[i][n] * f;
        }
    }
}

// weights of the splits of one query into LDS: exp2(m - max) / sum (zero for empty splits).  One wave.
__device__ __forceinline__ void split_weights(const float *__restrict__ ml, int64_t stride, int nz, float *wz, int lane) {
    float m = -INFINITY, l = 0.0f;
    for (int z = lane; z < nz; z += 64) m = fmaxf(m, ml[z * stride]);
    m = wave_max(m);
    for (int z = lane; z < nz; z += 64) {
        const float e = __builtin_amdgcn_exp2f(ml[z * stride] - m);
        wz[z] = e;
        l = fmaf(e, ml[z * stride + 1], l);
    }
    l = wave_sum(l);
    for (int z = lane; z < nz; z += 64) wz[z] /= l;
}

// The records of one query, merged: 256 threads as groups of n4 (float4 columns of the latent), group g on splits g, g + groups, ...  The first splits are on
// their way before the weights are known.  Leaves the sum in o (LDS, n4 float4; acc: groups * n4 float4).
constexpr int MAX_SPLITS = 256;
__device__ __forceinline__ void merge_latent(const float *__restrict__ part, int64_t stride, const float *__restrict__ ml, int64_t ml_stride, int nz, int n4, f32x4 *acc,
                                             f32x4 *o, float *wz) {
    const int tid = threadIdx.x, groups = 256 / n4, g = tid / n4, c = tid - g * n4;
    constexpr int U = 16;
    f32x4 v[U], a = {0.f, 0.f, 0.f, 0.f};
    const float *src = part + 4 * c;
#pragma unroll
    for (int i = 0; i < U; i++) v[i] = *reinterpret_cast<const f32x4 *>(src + min(g + i * groups, nz - 1) * stride);
    if (tid < 64) split_weights(ml, ml_stride, nz, wz, tid);
    __syncthreads();
    if (g < groups)
        for (int z0 = g; z0 < nz; z0 += U * groups) {
            if (z0 != g) {
#pragma unroll
                for (int i = 0; i < U; i++) v[i] = *reinterpret_cast<const f32x4 *>(src + min(z0 + i * groups, nz - 1) * stride);
            }
#pragma unroll
            for (int i = 0; i < U; i++) {
                const int z = z0 + i * groups;
                const float w = z < nz ? wz[z] : 0.0f;
#pragma unroll
                for (int e = 0; e < 4; e++) a[e] = w > 0.0f ? fmaf(w, v[i][e], a[e]) : a[e];       // an empty split has not written its record
            }
        }
    if (g < groups) acc[tid] = a;
    __syncthreads();
    if (tid < n4) {
        for (int i = 1; i < groups; i++) a += acc[tid + i * n4];
        o[tid] = a;
    }
    __syncthreads();
}

// one workgroup per query: the records of its splits into the gated latent
__global__ __launch_bounds__(256) void latent_combine_kernel(const float *__restrict__ part, int nz, int M, int heads, int rank_pad, const float *__restrict__ gate,
                                                             int64_t gate_row, float *__restrict__ out) {
    __shared__ float wz[MAX_SPLITS];
    __shared__ f32x4 acc[256], o[CQ_LATENT_MAX_RANK / 4];
    const int m = blockIdx.x;
    const float f = mix_sigmoid(gate[(m / heads) * gate_row + m % heads]);
    merge_latent(part + (int64_t)m * rank_pad, (int64_t)M * rank_pad, part + (int64_t)nz * M * rank_pad + 2 * m, 2 * (int64_t)M, nz, rank_pad >> 2, acc, o, wz);
    if ((int)threadIdx.x < rank_pad >> 2) *reinterpret_cast<f32x4 *>(out + (int64_t)m * rank_pad + 4 * threadIdx.x) = o[threadIdx.x] * f;
}

// ---- projection rows into queries and cache rows -----------------------------------------------------------------------------------------------
__device__ __forceinline__ float query_factor(const cq_latent &g) { return g.scale * 1.44269504088896341f; }

template <typename T> __device__ __forceinline__ float turned(const cq_latent &g, const float *src, int64_t p, int d) {
    const int half = g.rot_dim >> 1;
    const float c = g.cos_dev[p * half + (d >> 1)], s = g.sin_dev[p * half + (d >> 1)], v = src[d], w = src[d ^ 1];
    return d & 1 ? v * c + w * s : v * c - w * s;
}

// latent (normed) and rotated key part of one projection row into the cache row of position p; all threads of the workgroup
template <typename T, int THREADS> __device__ __forceinline__ void append_row(const cq_latent &g, const float *src, T *dst, int64_t p, float *red) {
    const int tid = threadIdx.x, lane = tid & 63;
    float q = 0.0f;
    for (int i = tid; i < g.rank; i += THREADS) q = fmaf(src[i], src[i], q);
    q = wave_sum(q);
    if (lane == 0) red[tid >> 6] = q;
    __syncthreads();
    q = 0.0f;
#pragma unroll
    for (int i = 0; i < THREADS / 64; i++) q += red[i];
    const float m = sqrtf(q / (float)g.rank + g.eps);
    for (int i = tid; i < g.rank; i += THREADS) dst[i] = (T)(src[i] / m * g.norm_dev[i]);
    for (int d = tid; d < g.rot_dim; d += THREADS) dst[g.rank_pad + d] = (T)turned<T>(g, src + g.rank, p, d);
}

// One workgroup per row.  plain != nullptr: unrotated query dimensions go there as f32, [row][head][plain_head]; else to the front of the head in q.
template <typename T>
__global__ __launch_bounds__(256) void latent_pack_kernel(cq_latent g, const float *__restrict__ row, int64_t row_stride, int64_t kv_off, T *cache, float *plain,
                                                          int plain_head, T *q, int q_head, int rot_off, int64_t pos) {
    __shared__ float red[4];
    const int64_t r = blockIdx.x, p = pos + r;
    const float *src = row + r * row_stride;
    const int lane = threadIdx.x & 63, dq = g.dim + g.rot_dim;
    const float fq = query_factor(g);
    for (int h = threadIdx.x >> 6; h < g.heads; h += 4) {
        const float *s = src + (int64_t)h * dq;
        T *d = q + (r * g.heads + h) * q_head;
        float *f = plain ? plain + (r * g.heads + h) * plain_head : nullptr;
        for (int i = lane; i < g.dim; i += 64) {
            if (f) f[i] = fq * s[i];
            else d[i] = (T)(fq * s[i]);
        }
        if (!f)
            for (int i = g.dim + lane; i < rot_off; i += 64) d[i] = (T)0.0f;
        for (int i = lane; i < q_head - rot_off; i += 64) d[rot_off + i] = i < g.rot_dim ? (T)(fq * turned<T>(g, s + g.dim, p, i)) : (T)0.0f;
    }
    if (kv_off >= 0) append_row<T, 256>(g, src + kv_off, cache + p * (g.rank_pad + g.rot_pad), p, red);
}

// One token: workgroup (head, 64 latent columns) takes W_uk of its head to the query; those of the first columns rotate the rest of it.  The last workgroup
// appends the cache row.  w_ukt [head][rank][ldw]: row j is column j of W_uk.
template <typename T>
__global__ __launch_bounds__(256) void latent_absorb_step_kernel(cq_latent g, const float *__restrict__ row, int64_t kv_off, T *cache, const uint16_t *__restrict__ w_ukt,
                                                                 int ldw, T *__restrict__ q, const int32_t *__restrict__ pos_dev, int pos0) {
    __shared__ float red[4];
    const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, sub = lane & 15, dq = g.dim + g.rot_dim, ld = g.rank_pad + g.rot_pad;
    const int pieces = (g.rank + 63) / 64, h = blockIdx.x / pieces, piece = blockIdx.x % pieces;
    const int64_t p = pos0 + (pos_dev ? pos_dev[0] : 0);
    if (p >= g.ctx) return;
    if (h == g.heads) {
        if (kv_off >= 0) append_row<T, 256>(g, row + kv_off, cache + p * ld, p, red);
        return;
    }
    const float *s = row + (int64_t)h * dq;
    T *d = q + (int64_t)h * ld;
    const int j0 = piece * 64 + wv * 16 + (lane >> 4);
    const uint16_t *w = w_ukt + (int64_t)h * g.rank * ldw;
    float acc[4][2] = {};
    for (int c0 = 0; c0 < g.dim; c0 += 128) {
        const int c = c0 + 8 * sub;
        u32x4 wr[4];
#pragma unroll
        for (int i = 0; i < 4; i++) wr[i] = c < ldw ? *reinterpret_cast<const u32x4 *>(w + (int64_t)min(j0 + 4 * i, g.rank - 1) * ldw + c) : u32x4{0, 0, 0, 0};
        f32x4 a, b;
#pragma unroll
        for (int e = 0; e < 4; e++) {
            a[e] = c + e < g.dim ? s[c + e] : 0.0f;
            b[e] = c + 4 + e < g.dim ? s[c + 4 + e] : 0.0f;
        }
#pragma unroll
        for (int i = 0; i < 4; i++) dot8(wr[i], a, b, acc[i]);
    }
#pragma unroll
    for (int i = 0; i < 4; i++) {
        const float v = row16_sum(acc[i][0] + acc[i][1]);
        if (sub == 0 && j0 + 4 * i < g.rank) d[j0 + 4 * i] = (T)(query_factor(g) * v);
    }
    if (piece == 0)
        for (int i = threadIdx.x; i < g.rot_pad; i += 256) d[g.rank_pad + i] = i < g.rot_dim ? (T)(query_factor(g) * turned<T>(g, s + g.dim, p, i)) : (T)0.0f;
}

// One token: workgroup (head, 16 value rows) merges the records of the head's splits and takes W_uv to the latent.
__global__ __launch_bounds__(256) void latent_merge_step_kernel(const float *__restrict__ part, int nz, int heads, int rank_pad, const uint16_t *__restrict__ w_uv, int ldw,
                                                                const float *__restrict__ gate, float *__restrict__ out, int vdim) {
    __shared__ float wz[MAX_SPLITS];
    __shared__ f32x4 acc[256], o[CQ_LATENT_MAX_RANK / 4];
    const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, h = blockIdx.x, e0 = blockIdx.y * 16 + 4 * wv;
    u32x4 wr[4];
#pragma unroll
    for (int i = 0; i < 4; i++) wr[i] = *reinterpret_cast<const u32x4 *>(w_uv + ((int64_t)h * vdim + min(e0 + i, vdim - 1)) * ldw + min(8 * lane, ldw - 8));
    const float g = gate[h];
    merge_latent(part + (int64_t)h * rank_pad, (int64_t)heads * rank_pad, part + (int64_t)nz * heads * rank_pad + 2 * h, 2 * (int64_t)heads, nz, rank_pad >> 2, acc, o, wz);
    float s[4][2] = {};
    if (8 * lane < rank_pad) {                             // rank_pad <= 512: one piece per lane
        const f32x4 a = o[2 * lane], b = o[2 * lane + 1];
#pragma unroll
        for (int i = 0; i < 4; i++) dot8(wr[i], a, b, s[i]);
    }
#pragma unroll
    for (int i = 0; i < 4; i++) {
        const float v = wave_sum(s[i][0] + s[i][1]);
        if (lane == 0 && e0 + i < vdim) out[h * vdim + e0 + i] = v * mix_sigmoid(g);
    }
}

int check_latent(const cq_latent *g) {
    if (!g) return CQ_ERR_NULL;
    if (g->heads <= 0 || g->dim <= 0 || g->vdim <= 0 || g->rank <= 0 || g->rot_dim < 0 || g->rot_dim % 2 || g->ctx <= 0 || g->rank_pad < g->rank || g->rank_pad % 64 ||
        g->rot_pad < g->rot_dim || g->rot_pad % 8)
        return CQ_ERR_SHAPE;
    if (g->rot_dim && (!g->cos_dev || !g->sin_dev)) return CQ_ERR_NULL;
    if (g->rot_pad > 192 || g->rank_pad > (g->rot_pad > 64 ? 256 : CQ_LATENT_MAX_RANK) || g->heads > 4096 || g->dim > 4096 || g->vdim > 4096 || g->ctx > (1 << 24))
        return CQ_ERR_RANGE;
    return CQ_OK;
}

// Queries per workgroup (in 16s) and splits of the keys: 16 while all (block of queries, tile of keys) pairs can run side by side.
struct AbsorbedPlan {
    int nq, splits;
};
AbsorbedPlan absorbed_plan(int bf16, int64_t m, int64_t keys) {
    const int64_t kt = bf16 ? 64 : 32, tiles = (keys + kt - 1) / kt, fine = (m + 15) / 16;
    AbsorbedPlan p;
    p.nq = bf16 && fine > 1 && fine * tiles > 256 ? 2 : 1;
    const int64_t blocks = (m + 16 * p.nq - 1) / (16 * p.nq);
    int64_t n = blocks >= 256 ? 1 : 256 / blocks;
    n = n < tiles ? n : tiles;
    p.splits = (int)(n < MAX_SPLITS ? n : MAX_SPLITS);
    return p;
}

template <typename T, int DV, int DR, int NQ> int absorbed_launch(const Absorbed &a, int nz, hipStream_t s) {
    constexpr size_t lds = (size_t)Chunk<T>::KEYS * (DV + DR) * sizeof(T) + (size_t)DV * 128 + (size_t)2 * 16 * NQ * (Chunk<T>::KEYS + 4) * sizeof(float);
    static_assert(lds <= (size_t)160 * 1024, "LDS");
    if (lds > 64 * 1024) {
        const int e = (int)hipFuncSetAttribute(reinterpret_cast<const void *>(latent_absorbed_kernel<T, DV, DR, NQ>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e) return e;
    }
    hipLaunchKernelGGL((latent_absorbed_kernel<T, DV, DR, NQ>), dim3((unsigned)((a.rows * a.heads + 16 * NQ - 1) / (16 * NQ)), 1, nz), dim3(256), lds, s, a);
    return (int)hipGetLastError();
}
template <typename T> int absorbed_dispatch(const Absorbed &a, const AbsorbedPlan &plan, hipStream_t s) {
    const int nz = plan.splits;
#define CQ_AB(DV_, DR_)                                                                                                                              \
    do {                                                                                                                                             \
        if constexpr (sizeof(T) == 2) {                                                                                                              \
            if (plan.nq == 2) return absorbed_launch<T, DV_, DR_, 2>(a, nz, s);                                      \
        }                                                                                                                                            \
        return absorbed_launch<T, DV_, DR_, 1>(a, nz, s);                                                                                            \
    } while (0)
    if (a.ld - a.rank_pad > 64) CQ_AB(256, 192);
    if (a.rank_pad <= 128) CQ_AB(128, 64);
    if (a.rank_pad <= 256) CQ_AB(256, 64);
    CQ_AB(512, 64);
#undef CQ_AB
}

template <typename T, int DK, int DV, int NQ> int expanded_launch(const Expanded &a, hipStream_t s) {
    const int64_t blocks = (int64_t)((a.rows + 64 * NQ - 1) / (64 * NQ)) * a.heads;
    if (blocks > 0x7fffffffLL) return CQ_ERR_RANGE;
    hipLaunchKernelGGL((latent_expanded_kernel<T, DK, DV, NQ>), dim3((unsigned)blocks), dim3(256), 0, s, a);
    return (int)hipGetLastError();
}

}  // namespace

extern "C" {

int cq_mix_latent_pack(const cq_latent *g, const float *row_dev, int64_t row_stride, int64_t kv_off, void *cache_dev, float *plain_dev, int64_t plain_head, void *q_dev,
                       int64_t q_head, int64_t rot_off, int64_t pos, int64_t rows, void *stream) {
    const int e = check_latent(g);
    if (e) return e;
    const int64_t dq = g->dim + g->rot_dim;
    if (rows < 0 || pos < 0 || row_stride < g->heads * dq || (kv_off >= 0 && kv_off + g->rank + g->rot_dim > row_stride) || q_head < rot_off + g->rot_dim ||
        (plain_dev ? plain_head < g->dim : rot_off < g->dim))
        return CQ_ERR_SHAPE;
    if (rows == 0) return CQ_OK;
    if (!row_dev || !q_dev || (kv_off >= 0 && (!cache_dev || !g->norm_dev))) return CQ_ERR_NULL;
    if (pos + rows > g->ctx || q_head > (1 << 20)) return CQ_ERR_RANGE;
#define CQ_LP(T_) hipLaunchKernelGGL(latent_pack_kernel<T_>, dim3((unsigned)rows), dim3(256), 0, (hipStream_t)stream, *g, row_dev, row_stride, kv_off, (T_ *)cache_dev, \
                                     plain_dev, (int)plain_head, (T_ *)q_dev, (int)q_head, (int)rot_off, pos)
    if (g->bf16) CQ_LP(__bf16);
    else CQ_LP(float);
#undef CQ_LP
    return (int)hipGetLastError();
}

int cq_mix_latent_expanded(const cq_latent *g, const void *q_dev, int64_t dim_pad, const void *kv_dev, int64_t kv_row, int64_t v_off, int64_t v_pad, const void *cache_dev,
                           const float *gate_dev, int64_t gate_row, void *out_dev, int64_t out_row, int64_t pos, int64_t rows, void *stream) {
    const int e = check_latent(g);
    if (e) return e;
    if (rows < 0 || pos < 0 || dim_pad < g->dim || dim_pad % 8 || v_pad < g->vdim || v_pad % 8 || v_off % 8 || kv_row % 8 || v_off < g->heads * dim_pad ||
        kv_row < v_off + g->heads * v_pad || gate_row < g->heads || out_row < g->heads * g->vdim)
        return CQ_ERR_SHAPE;
    if (rows == 0) return CQ_OK;
    if (!q_dev || !kv_dev || !cache_dev || !gate_dev || !out_dev) return CQ_ERR_NULL;
    if (misaligned(q_dev, 16) || misaligned(kv_dev, 16) || misaligned(cache_dev, 16) || misaligned(out_dev, 16)) return CQ_ERR_ALIGN;
    if (pos + rows > g->ctx || dim_pad + g->rot_pad > CQ_LATENT_MAX_HEAD || v_pad > CQ_LATENT_MAX_VALUE) return CQ_ERR_RANGE;
    Expanded a;
    const size_t el = g->bf16 ? 2 : 4;
    a.q = q_dev;
    a.k = kv_dev;
    a.kr = (const char *)cache_dev + el * g->rank_pad;
    a.v = (const char *)kv_dev + el * v_off;
    a.q_head = (int)(dim_pad + g->rot_pad);
    a.q_row = (int64_t)g->heads * a.q_head;
    a.k_row = a.v_row = kv_row;
    a.kr_row = g->rank_pad + g->rot_pad;
    a.k_head = a.d1 = (int)dim_pad;
    a.d2 = g->rot_pad;
    a.v_head = a.v_pad = (int)v_pad;
    a.vdim = g->vdim;
    a.gate = gate_dev;
    a.gate_row = gate_row;
    a.out = out_dev;
    a.out_row = out_row;
    a.pos = (int)pos;
    a.rows = (int)rows;
    a.heads = g->heads;
    hipStream_t s = (hipStream_t)stream;
    const int dk = a.q_head;
    // 32 query rows per wave where that leaves two workgroups per CU
    const bool wide = (rows + 127) / 128 * g->heads >= 512;
#define CQ_EX(DK_, DV_)                                                                                                     \
    do {                                                                                                                    \
        if (!g->bf16) return expanded_launch<float, DK_, DV_, 1>(a, s);                                                     \
        return wide ? expanded_launch<__bf16, DK_, DV_, 2>(a, s) : expanded_launch<__bf16, DK_, DV_, 1>(a, s);              \
    } while (0)
    if (dk <= 128 && v_pad <= 128) CQ_EX(128, 128);
    if (dk <= 192 && v_pad <= 128) CQ_EX(192, 128);
    return g->bf16 ? expanded_launch<__bf16, 320, 256, 1>(a, s) : expanded_launch<float, 320, 256, 1>(a, s);
#undef CQ_EX
}

int64_t cq_mix_latent_absorbed_workspace_bytes(const cq_latent *g, int64_t rows, int64_t pos, int step) {
    if (check_latent(g) || rows <= 0) return -1;
    const int64_t m = rows * g->heads;
    const int nz = absorbed_plan(g->bf16, m, step ? g->ctx : pos + rows).splits;
    return nz > 1 || step ? nz * m * (g->rank_pad + 2) * 4 : 0;
}

int cq_mix_latent_absorbed(const cq_latent *g, const void *q_dev, const void *cache_dev, const float *gate_dev, int64_t gate_row, float *out_dev, int64_t pos, int64_t rows,
                           void *workspace_dev, int64_t workspace_bytes, void *stream) {
    const int e = check_latent(g);
    if (e) return e;
    if (rows < 0 || pos < 0 || gate_row < g->heads) return CQ_ERR_SHAPE;
    if (rows == 0) return CQ_OK;
    if (!q_dev || !cache_dev || !gate_dev || !out_dev) return CQ_ERR_NULL;
    if (misaligned(q_dev, 16) || misaligned(cache_dev, 16) || misaligned(out_dev, 16) || misaligned(workspace_dev, 16)) return CQ_ERR_ALIGN;
    if (pos + rows > g->ctx || rows * g->heads > (1 << 24)) return CQ_ERR_RANGE;
    const int64_t m = rows * g->heads, need = cq_mix_latent_absorbed_workspace_bytes(g, rows, pos, 0);
    const AbsorbedPlan plan = absorbed_plan(g->bf16, m, pos + rows);
    const int nz = plan.splits;
    if (need && (!workspace_dev || workspace_bytes < need)) return CQ_ERR_WORKSPACE;
    Absorbed a;
    a.q = q_dev;
    a.cache = cache_dev;
    a.ld = g->rank_pad + g->rot_pad;
    a.rank_pad = g->rank_pad;
    a.heads = g->heads;
    a.rows = (int)rows;
    a.pos = (int)pos;
    a.ctx = g->ctx;
    a.pos_dev = nullptr;
    a.gate = gate_dev;
    a.gate_row = gate_row;
    a.out = out_dev;
    a.part = nz > 1 ? (float *)workspace_dev : nullptr;
    hipStream_t s = (hipStream_t)stream;
    const int r = g->bf16 ? absorbed_dispatch<__bf16>(a, plan, s) : absorbed_dispatch<float>(a, plan, s);
    if (r || nz == 1) return r;
    hipLaunchKernelGGL(latent_combine_kernel, dim3((unsigned)m), dim3(256), 0, s, (const float *)workspace_dev, nz, (int)m, g->heads, g->rank_pad, gate_dev, gate_row, out_dev);
    return (int)hipGetLastError();
}

int cq_mix_latent_step(const cq_latent *g, const float *row_dev, int64_t kv_off, void *cache_dev, const void *w_ukt_dev, int64_t ld_ukt, const void *w_uv_dev, int64_t ld_uv,
                       int64_t gate_off, void *q_dev, float *out_dev, const int32_t *pos_dev, int64_t pos, void *workspace_dev, int64_t workspace_bytes, void *stream) {
    const int e = check_latent(g);
    if (e) return e;
    if (pos < 0 || ld_ukt < g->dim || ld_ukt % 8 || ld_uv < g->rank_pad || ld_uv % 8 || gate_off < 0) return CQ_ERR_SHAPE;
    if (!row_dev || !cache_dev || !w_ukt_dev || !w_uv_dev || !q_dev || !out_dev || !workspace_dev || (kv_off >= 0 && !g->norm_dev)) return CQ_ERR_NULL;
    if (misaligned(cache_dev, 16) || misaligned(w_ukt_dev, 16) || misaligned(w_uv_dev, 16) || misaligned(q_dev, 16) || misaligned(workspace_dev, 16)) return CQ_ERR_ALIGN;
    if (pos >= g->ctx) return CQ_ERR_RANGE;
    if (workspace_bytes < cq_mix_latent_absorbed_workspace_bytes(g, 1, 0, 1)) return CQ_ERR_WORKSPACE;
    const AbsorbedPlan plan = absorbed_plan(g->bf16, g->heads, g->ctx);
    const int nz = plan.splits;
    hipStream_t s = (hipStream_t)stream;
    const dim3 grid((unsigned)(g->heads * ((g->rank + 63) / 64) + 1));
    if (g->bf16)
        hipLaunchKernelGGL(latent_absorb_step_kernel<__bf16>, grid, dim3(256), 0, s, *g, row_dev, kv_off, (__bf16 *)cache_dev, (const uint16_t *)w_ukt_dev, (int)ld_ukt,
                           (__bf16 *)q_dev, pos_dev, (int)pos);
    else
        hipLaunchKernelGGL(latent_absorb_step_kernel<float>, grid, dim3(256), 0, s, *g, row_dev, kv_off, (float *)cache_dev, (const uint16_t *)w_ukt_dev, (int)ld_ukt,
                           (float *)q_dev, pos_dev, (int)pos);
    Absorbed a = {};
    a.q = q_dev;
    a.cache = cache_dev;
    a.ld = g->rank_pad + g->rot_pad;
    a.rank_pad = g->rank_pad;
    a.heads = g->heads;
    a.rows = 1;
    a.pos = (int)pos;
    a.ctx = g->ctx;
    a.pos_dev = pos_dev;
    a.part = (float *)workspace_dev;
    const int r = g->bf16 ? absorbed_dispatch<__bf16>(a, plan, s) : absorbed_dispatch<float>(a, plan, s);
    if (r) return r;
    hipLaunchKernelGGL(latent_merge_step_kernel, dim3((unsigned)g->heads, (unsigned)((g->vdim + 15) / 16)), dim3(256), 0, s,
                       (const float *)workspace_dev, nz, g->heads, g->rank_pad, (const uint16_t *)w_uv_dev, (int)ld_uv, row_dev + gate_off, out_dev, g->vdim);
    return (int)hipGetLastError();
}

}  // extern "C"
