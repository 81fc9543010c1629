// Sequence mixers with a recurrent matrix state per head: linear attention with a fixed decay (retention) and the generalized
// delta rule.  States are f32 and stored by columns, [head][value column][state_pad]: a wave holds four columns with 16 lanes
// on the rows of each, so a step over one token needs 16-lane sums only.
#include "cq_mix.h"

namespace {

// ---- retention, several tokens ----------------------------------------------------------------------------------------------
// Chunks of 64 tokens on v_mfma_f32_16x16x4; workgroup: 4 waves on one head and 64 value columns.  With gamma the head's decay, i and j
// places in the chunk and S the state before it:
//   o_i = gamma^(i+1) S^T q_i + sum_{j<=i} gamma^(i-j) (q_i . k_j) v_j,     S' = gamma^n S + sum_j gamma^(n-1-j) k_j v_j^T
// A long call is cut into segments of whole chunks that run side by side: retention_segment_kernel leaves what each segment adds to the
// state (Z), retention_prefix_kernel turns Z into the state before each segment and forms the final one.
constexpr int RC = 64, RLD = 68;                     // chunk length; LDS row of 64 columns (16 rows x 4 fall on 64 banks)

struct Retention {
    const float *q, *k, *v, *log2_decay;
    float *state, *out, *z;
    int64_t v_stride, out_stride;
    int rows, heads, dp, vdim, sp, nvb, nseg, seg_len;      // sp: state_pad
};

__device__ __forceinline__ float *segment_z(const Retention &a, int h, int vb, int seg) {
    return a.z + (((int64_t)h * a.nvb + vb) * a.nseg + seg) * a.dp * 64;
}

// V of a chunk as operand: vf[s][n] = v[t0 + 4 s + lk][64 vb + 16 n + lr] (rows beyond the chunk repeat its last one: their weights are zero)
__device__ __forceinline__ void load_v(const Retention &a, int h, int vb, int t0, int n_tok, int lr, int lk, float (&vf)[16][4]) {
#pragma unroll
    for (int s = 0; s < 16; s++) {
        const float *vr = a.v + (int64_t)(t0 + min(4 * s + lk, n_tok - 1)) * a.v_stride + (int64_t)h * a.vdim;
#pragma unroll
        for (int n = 0; n < 4; n++) vf[s][n] = vr[min(64 * vb + 16 * n + lr, a.vdim - 1)];
    }
}

// acc[n] += sum_j gamma^(n_tok-1-j) k_j[16 dt + lr ...] v_j[...] over the chunk
__device__ __forceinline__ void add_kv(const Retention &a, int h, int dt, int t0, int n_tok, float l2, int lr, int lk, const float (&vf)[16][4],
                                       f32x4 (&acc)[4]) {
    float kf[16];
#pragma unroll
    for (int s = 0; s < 16; s++) kf[s] = a.k[((int64_t)(t0 + min(4 * s + lk, n_tok - 1)) * a.heads + h) * a.dp + 16 * dt + lr];
#pragma unroll
    for (int s = 0; s < 16; s++) {
        const int j = 4 * s + lk;
        const float kw = j < n_tok ? kf[s] * exp2f(l2 * (float)(n_tok - 1 - j)) : 0.0f;
#pragma unroll
        for (int n = 0; n < 4; n++) acc[n] = mfma4(kw, vf[s][n], acc[n]);
    }
}

__global__ __launch_bounds__(256) void retention_segment_kernel(Retention a) {
    const int tid = threadIdx.x, lane = tid & 63, wv = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lk = lane >> 4;
    const int h = blockIdx.x / a.nvb, vb = blockIdx.x % a.nvb, seg = blockIdx.y;
    const float l2 = a.log2_decay[h];
    const int t_end = min(a.rows, (seg + 1) * a.seg_len);
    float *z = segment_z(a, h, vb, seg);
    for (int dt = wv; dt < a.dp / 16; dt += 4) {
        f32x4 acc[4];
#pragma unroll
        for (int n = 0; n < 4; n++) acc[n] = f32x4{0.f, 0.f, 0.f, 0.f};
        for (int t0 = seg * a.seg_len; t0 < t_end; t0 += RC) {
            const int n_tok = min(RC, t_end - t0);
            float vf[16][4];
            load_v(a, h, vb, t0, n_tok, lr, lk, vf);
            const float g = exp2f(l2 * (float)n_tok);
#pragma unroll
            for (int n = 0; n < 4; n++) acc[n] *= g;
            add_kv(a, h, dt, t0, n_tok, l2, lr, lk, vf, acc);
        }
#pragma unroll
        for (int n = 0; n < 4; n++)
#pragma unroll
            for (int e = 0; e < 4; e++) z[(16 * dt + 4 * lk + e) * 64 + 16 * n + lr] = acc[n][e];
    }
}

__global__ __launch_bounds__(256, 2) void retention_kernel(Retention a) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    float *S = smem, *A = S + a.dp * RLD;                 // state [dp][64], decayed q k^T [64][64]
    const int tid = threadIdx.x, lane = tid & 63, wv = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lk = lane >> 4;
    const int h = blockIdx.x / a.nvb, vb = blockIdx.x % a.nvb, seg = blockIdx.y;
    const float l2 = a.log2_decay[h];
    const int seg0 = seg * a.seg_len, t_end = min(a.rows, seg0 + a.seg_len);
    float *state = a.state + (int64_t)h * a.vdim * a.sp;

    if (a.nseg > 1) {
        const float *z = segment_z(a, h, vb, seg);
        for (int i = tid; i < a.dp * 64; i += 256) S[(i >> 6) * RLD + (i & 63)] = z[i];
    } else {
        for (int i = tid; i < a.dp * 64; i += 256) {
            const int col = i / a.dp, d = i - col * a.dp;      // rows of a column follow each other in memory
            S[d * RLD + col] = 64 * vb + col < a.vdim ? state[(int64_t)(64 * vb + col) * a.sp + d] : 0.0f;
        }
    }
    __syncthreads();

    const int n_d = a.dp / 16;
    for (int t0 = seg0; t0 < t_end; t0 += RC) {
        const int n_tok = min(RC, t_end - t0);
        float vf[16][4];
        load_v(a, h, vb, t0, n_tok, lr, lk, vf);
        // rows 16 wv .. of the chunk: A and S^T q
        f32x4 sc[4], o[4];
#pragma unroll
        for (int n = 0; n < 4; n++) sc[n] = o[n] = f32x4{0.f, 0.f, 0.f, 0.f};
        const float *qr = a.q + ((int64_t)(t0 + min(16 * wv + lr, n_tok - 1)) * a.heads + h) * a.dp + 4 * lk;
        const float *kr[4];
#pragma unroll
        for (int n = 0; n < 4; n++) kr[n] = a.k + ((int64_t)(t0 + min(16 * n + lr, n_tok - 1)) * a.heads + h) * a.dp + 4 * lk;
        for (int c = 0; c < n_d; c++) {
            const f32x4 qf = *reinterpret_cast<const f32x4 *>(qr + 16 * c);
            f32x4 kf[4];
#pragma unroll
            for (int n = 0; n < 4; n++) kf[n] = *reinterpret_cast<const f32x4 *>(kr[n] + 16 * c);
#pragma unroll
            for (int e = 0; e < 4; e++)
#pragma unroll
                for (int n = 0; n < 4; n++) {
                    if (n <= wv) sc[n] = mfma4(qf[e], kf[n][e], sc[n]);
                    o[n] = mfma4(qf[e], S[(16 * c + 4 * lk + e) * RLD + 16 * n + lr], o[n]);
                }
        }
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int i = 16 * wv + 4 * lk + e;
            const float g = exp2f(l2 * (float)(i + 1));
#pragma unroll
            for (int n = 0; n < 4; n++) {
                o[n][e] *= g;
                const int j = 16 * n + lr;
                A[i * RLD + j] = j <= i && j < n_tok ? sc[n][e] * exp2f(l2 * (float)(i - j)) : 0.0f;
            }
        }
        __syncthreads();                                    // A is written, and every wave has read S
#pragma unroll
        for (int s = 0; s < 16; s++)
            if (s < 4 * (wv + 1)) {
                const float w = A[(16 * wv + lr) * RLD + 4 * s + lk];
#pragma unroll
                for (int n = 0; n < 4; n++) o[n] = mfma4(w, vf[s][n], o[n]);
            }
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int i = 16 * wv + 4 * lk + e;
            if (i >= n_tok) continue;
#pragma unroll
            for (int n = 0; n < 4; n++) {
                const int col = 64 * vb + 16 * n + lr;
                if (col < a.vdim) a.out[(int64_t)(t0 + i) * a.out_stride + (int64_t)h * a.vdim + col] = o[n][e];
            }
        }
        if (t0 + RC < t_end || a.nseg == 1) {
            const float g = exp2f(l2 * (float)n_tok);
            for (int dt = wv; dt < n_d; dt += 4) {
                f32x4 acc[4];
#pragma unroll
                for (int n = 0; n < 4; n++)
#pragma unroll
                    for (int e = 0; e < 4; e++) acc[n][e] = g * S[(16 * dt + 4 * lk + e) * RLD + 16 * n + lr];
                add_kv(a, h, dt, t0, n_tok, l2, lr, lk, vf, acc);
#pragma unroll
                for (int n = 0; n < 4; n++)
#pragma unroll
                    for (int e = 0; e < 4; e++) S[(16 * dt + 4 * lk + e) * RLD + 16 * n + lr] = acc[n][e];
            }
        }
        __syncthreads();
    }
    if (a.nseg == 1)
        for (int i = tid; i < a.dp * 64; i += 256) {
            const int col = i / a.dp, d = i - col * a.dp;
            if (64 * vb + col < a.vdim) state[(int64_t)(64 * vb + col) * a.sp + d] = S[d * RLD + col];
        }
}

__global__ __launch_bounds__(256) void retention_prefix_kernel(Retention a) {
    const int h = blockIdx.y;
    const int i = blockIdx.x * 256 + threadIdx.x;             // element of the [nvb][dp][64] Z of a segment
    if (i >= a.nvb * a.dp * 64) return;
    const int vb = i / (a.dp * 64), in = i - vb * a.dp * 64, d = in >> 6, col = 64 * vb + (in & 63);
    const float l2 = a.log2_decay[h], g = exp2f(l2 * (float)a.seg_len), g_last = exp2f(l2 * (float)(a.rows - (a.nseg - 1) * a.seg_len));
    float *st = a.state + ((int64_t)h * a.vdim + min(col, a.vdim - 1)) * a.sp + d;
    float *z = segment_z(a, h, vb, 0) + in;
    const int64_t step = (int64_t)a.dp * 64;
    float s = col < a.vdim ? st[0] : 0.0f;
    constexpr int B = 8;                                      // the loads of eight segments before their chain
    for (int x0 = 0; x0 < a.nseg; x0 += B) {
        float v[B];
#pragma unroll
        for (int x = 0; x < B; x++) v[x] = z[min(x0 + x, a.nseg - 1) * step];
#pragma unroll
        for (int x = 0; x < B; x++)
            if (x0 + x < a.nseg) {
                z[(x0 + x) * step] = s;
                s = fmaf(x0 + x == a.nseg - 1 ? g_last : g, s, v[x]);
            }
    }
    if (col < a.vdim) st[0] = s;
}

void retention_plan(int64_t rows, int64_t heads, int64_t vdim, int *nseg, int *seg_len) {
    const int64_t wg = heads * ((vdim + 63) / 64), chunks = (rows + RC - 1) / RC;
    int64_t n = 512 / wg;
    n = n < chunks / 2 ? n : chunks / 2;                   // at least two chunks per segment
    n = n < 1 ? 1 : n;
    const int64_t per = (chunks + n - 1) / n;
    *seg_len = (int)(per * RC);
    *nseg = (int)((rows + *seg_len - 1) / *seg_len);
}

// ---- one token: merge of the attention records, and the retention step --------------------------------------------------------
struct StepArgs {
    const float *rec;
    int n_head, att_vdim, window, keep_first, ctx, splits, split_keys;
    float att_scale, ret_scale, eps;
    float *att_out, *state, *ret_out;
    const float *row, *decay;
    cq_mix_heads gq, gk;
    int64_t v_off, g_off;
    int heads, vdim;
};

// The state columns of a wave are requested before q and k are worked out.
template <int NR>
__device__ __forceinline__ void retention_step(const StepArgs &a, int h, int p, float *sm) {
    const int tid = threadIdx.x, lane = tid & 63, wv = __builtin_amdgcn_readfirstlane(tid >> 6), sub = lane & 15, cg = lane >> 4;
    constexpr int SP = 64 * NR;
    float *qs = sm, *ks = qs + SP, *os = ks + SP;
    __shared__ float s_inv;
    f32x4 s[NR];
    float vj;
    auto load = [&](int c0) {
        const int col = min(c0 + cg, a.vdim - 1);
        const float *st = a.state + ((int64_t)h * a.vdim + col) * SP + 4 * sub;
#pragma unroll
        for (int c = 0; c < NR; c++) s[c] = *reinterpret_cast<const f32x4 *>(st + 64 * c);
        vj = a.row[a.v_off + (int64_t)h * a.vdim + col];
    };
    load(4 * wv);
    if (wv < 2) {
        const cq_mix_heads &g = wv == 0 ? a.gq : a.gk;
        HeadShared<NR> sh;
        HeadRegs<NR> x;
        sh.load(g, p, lane);
        x.load(g, a.row + g.src_off + (int64_t)h * g.dim, lane);
        sh.ready(g, lane);
        x.finish(g, sh, a.eps, lane);
#pragma unroll
        for (int e = 0; e < NR; e++) sm[wv * SP + lane + 64 * e] = x.v[e];
    }
    const float dec = a.decay[h];
    __syncthreads();
    f32x4 qv[NR], kv[NR];
#pragma unroll
    for (int c = 0; c < NR; c++) {
        qv[c] = *reinterpret_cast<const f32x4 *>(qs + 64 * c + 4 * sub);
        kv[c] = *reinterpret_cast<const f32x4 *>(ks + 64 * c + 4 * sub);
    }
    for (int c0 = 4 * wv; c0 < a.vdim; c0 += 64) {
        if (c0 >= 64) load(c0);
        float o = 0.0f;
#pragma unroll
        for (int c = 0; c < NR; c++)
#pragma unroll
            for (int e = 0; e < 4; e++) {
                s[c][e] = fmaf(dec, s[c][e], kv[c][e] * vj);
                o = fmaf(s[c][e], qv[c][e], o);
            }
        o = row16_sum(o);
        if (c0 + cg < a.vdim) {
            float *st = a.state + ((int64_t)h * a.vdim + c0 + cg) * SP + 4 * sub;
#pragma unroll
            for (int c = 0; c < NR; c++) *reinterpret_cast<f32x4 *>(st + 64 * c) = s[c];
            if (sub == 0) os[c0 + cg] = o;
        }
    }
    __syncthreads();
    if (wv == 0) {
        const float inv = head_inv_rms(os, a.vdim, a.eps, lane);
        if (lane == 0) s_inv = inv;
    }
    __syncthreads();
    for (int e = tid; e < a.vdim; e += 1024) {
        const float g = a.row[a.g_off + (int64_t)h * a.vdim + e];
        a.ret_out[(int64_t)h * a.vdim + e] = a.ret_scale * os[e] * s_inv * (g * mix_sigmoid(g));
    }
}

// Blocks [0, n_head): out of one attention head from its records; blocks behind them: one retention head each.
template <int NR>
__global__ __launch_bounds__(1024) void talk_merge_retention_kernel(StepArgs a, const int32_t *__restrict__ pos_dev, int pos0) {
    extern __shared__ __attribute__((aligned(16))) float sm[];          // max(splits + 1024, 2 * 64 NR + vdim)
    __shared__ float red[16];
    const int tid = threadIdx.x, lane = tid & 63, wv = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int p = pos0 + (pos_dev ? pos_dev[0] : 0);
    if (p >= a.ctx) return;
    if ((int)blockIdx.x >= a.n_head) {
        retention_step<NR>(a, blockIdx.x - a.n_head, p, sm);
        return;
    }
    const int h = blockIdx.x, stride = talk_record(a.att_vdim);
    const int n = (visible_keys(p, a.window, a.keep_first).n + a.split_keys - 1) / a.split_keys;      // splits that hold keys
    const float *rec = a.rec + (int64_t)h * a.splits * stride;
    float *wt = sm, *part = sm + (n + 3) / 4 * 4;
    float m = -INFINITY;
    for (int s = tid; s < n; s += 1024) m = fmaxf(m, wt[s] = rec[(int64_t)s * stride + stride - 4]);
    m = wave_max(m);
    if (lane == 0) red[wv] = m;
    __syncthreads();
    m = red[0];
#pragma unroll
    for (int w = 1; w < 16; w++) m = fmaxf(m, red[w]);
    float l = 0.0f;
    for (int s = tid; s < n; s += 1024) {                    // the thread's own wt entries
        const float w = __expf(wt[s] - m);
        wt[s] = w;
        l = fmaf(w, rec[(int64_t)s * stride + stride - 3], l);
    }
    l = wave_sum(l);
    __syncthreads();
    if (lane == 0) red[wv] = l;
    __syncthreads();
    l = 0.0f;
#pragma unroll
    for (int w = 0; w < 16; w++) l += red[w];
    // 64 columns at a time, the waves share out the splits
    for (int e0 = 0; e0 < a.att_vdim; e0 += 64) {
        const int e = min(e0 + lane, a.att_vdim - 1);
        float acc = 0.0f;
#pragma unroll 4
        for (int s = wv; s < n; s += 16) acc = fmaf(wt[s], rec[(int64_t)s * stride + e], acc);
        __syncthreads();
        part[wv * 64 + lane] = acc;
        __syncthreads();
        if (wv == 0 && e0 + lane < a.att_vdim) {
            float t = 0.0f;
#pragma unroll
            for (int w = 0; w < 16; w++) t += part[w * 64 + lane];
            a.att_out[(int64_t)h * a.att_vdim + e0 + lane] = a.att_scale * t / l;
        }
    }
}

// ---- generalized delta rule ---------------------------------------------------------------------------------------------------
constexpr float DELTA_UNIT_EPS = 1e-6f;              // inside the root of the unit key
constexpr float DELTA_DECAY = 0.60653065971263342f;  // exp(-1/2)

__device__ __forceinline__ float delta_decay(float wl, float w0) { return expf(-DELTA_DECAY * mix_sigmoid(wl + w0)); }

// One head of a token as four vectors of `sp` floats, w | a u | u | r, zero beyond dim, and |k| (k = |k| u).  One wave.
template <typename WL>
__device__ __forceinline__ void delta_pack(const float *r, const float *k, const float *al, WL wl, const float *w0, const float *ab, float *dst, float *k_norm, int dim,
                                           int sp, int lane) {
    float s = 0.0f;
    for (int d = lane; d < dim; d += 64) s = fmaf(k[d], k[d], s);
    const float norm = sqrtf(wave_sum(s) + DELTA_UNIT_EPS), inv = 1.0f / norm;
    if (lane == 0) k_norm[0] = norm;
    for (int d = lane; d < sp; d += 64) {
        const bool ok = d < dim;
        const float u = ok ? k[d] * inv : 0.0f;
        dst[d] = ok ? delta_decay(wl(d), w0[d]) : 0.0f;
        dst[sp + d] = ok ? mix_sigmoid(al[d] + ab[d]) * u : 0.0f;
        dst[2 * sp + d] = u;
        dst[3 * sp + d] = ok ? r[d] : 0.0f;
    }
}

__global__ __launch_bounds__(256) void delta_prep_kernel(const float *__restrict__ row, int64_t row_stride, int64_t r_off, int64_t k_off, int64_t a_off,
                                                         const float *__restrict__ wl, int64_t wl_stride, const float *__restrict__ w0,
                                                         const float *__restrict__ ab, float *__restrict__ packed, int64_t rows, int heads, int dim, int sp) {
    const int lane = threadIdx.x & 63, h = blockIdx.y * 4 + (threadIdx.x >> 6);
    if (h >= heads) return;
    const int64_t t = blockIdx.x, id = t * heads + h, hd = (int64_t)h * dim;
    const float *s = row + t * row_stride + hd, *w = wl + t * wl_stride + hd;
    delta_pack(s + r_off, s + k_off, s + a_off, [&](int d) { return w[d]; }, w0 + hd, ab + hd, packed + id * 4 * sp, packed + rows * heads * 4 * sp + id, dim, sp, lane);
}

// The rows of a column that a lane holds, and one token's vectors on them.
template <int NR>
struct DeltaRows {
    f32x4 w[NR], b[NR], u[NR], r[NR];
    __device__ __forceinline__ void load(const float *vec, int sub) {
#pragma unroll
        for (int c = 0; c < NR; c++) {
            const float *x = vec + 64 * c + 4 * sub;
            w[c] = *reinterpret_cast<const f32x4 *>(x);
            b[c] = *reinterpret_cast<const f32x4 *>(x + 64 * NR);
            u[c] = *reinterpret_cast<const f32x4 *>(x + 2 * 64 * NR);
            r[c] = *reinterpret_cast<const f32x4 *>(x + 3 * 64 * NR);
        }
    }
};

// One column step: s <- w s - b (u . s) + u v (v: the value times |k|); returns this lane's part of r . s.
template <int NR>
__device__ __forceinline__ float delta_column(f32x4 (&s)[NR], const DeltaRows<NR> &x, float v) {
    float x0 = 0.0f, x1 = 0.0f;
#pragma unroll
    for (int c = 0; c < NR; c++) {
        x0 = fmaf(x.u[c].x, s[c].x, x0);
        x1 = fmaf(x.u[c].y, s[c].y, x1);
        x0 = fmaf(x.u[c].z, s[c].z, x0);
        x1 = fmaf(x.u[c].w, s[c].w, x1);
    }
    const float us = row16_sum(x0 + x1);
    float o0 = 0.0f, o1 = 0.0f;
#pragma unroll
    for (int c = 0; c < NR; c++) {
#pragma unroll
        for (int e = 0; e < 4; e++) s[c][e] = fmaf(-x.b[c][e], us, fmaf(x.w[c][e], s[c][e], x.u[c][e] * v));
        o0 = fmaf(x.r[c].x, s[c].x, o0);
        o1 = fmaf(x.r[c].y, s[c].y, o1);
        o0 = fmaf(x.r[c].z, s[c].z, o0);
        o1 = fmaf(x.r[c].w, s[c].w, o1);
    }
    return o0 + o1;
}

// Token after token.  Workgroup: 16 value columns of one head, 4 waves x 4 columns; the packed vectors of TB tokens at a time go
// through LDS (double-buffered: the next block's loads are in flight while this one runs) and from there, one token ahead, into
// registers.  The lanes' parts of r . s are collected for the block and summed 16 tokens at a time, off the chain of state updates.
template <int NR, int TB>
__global__ __launch_bounds__(256) void delta_scan_kernel(const float *__restrict__ packed, const float *__restrict__ v, int64_t v_stride,
                                                         float *__restrict__ state, float *__restrict__ out, int64_t out_stride, int rows, int heads, int dim,
                                                         int ncb) {
    constexpr int SP = 64 * NR, VEC = 4 * SP, LOADS = TB * VEC / 4 / 256;
    static_assert(TB * VEC % 1024 == 0 && TB <= 16, "whole float4 per thread");
    extern __shared__ __attribute__((aligned(16))) float smem[];         // 2 x { packed [TB][VEC], v [TB][16] }
    const int tid = threadIdx.x, lane = tid & 63, wv = __builtin_amdgcn_readfirstlane(tid >> 6), sub = lane & 15, cg = lane >> 4;
    // workgroups of one head on one XCD (dealt round-robin): they read the same packed vectors
    const int hb = blockIdx.x / (8 * ncb), in = blockIdx.x % (8 * ncb);
    const int h = hb * 8 + in % 8, cb = in / 8;
    if (h >= heads) return;
    const int col = 16 * cb + 4 * wv + cg, colc = min(col, dim - 1);
    float *st = state + ((int64_t)h * dim + colc) * SP + 4 * sub;
    f32x4 s[NR];
#pragma unroll
    for (int c = 0; c < NR; c++) s[c] = *reinterpret_cast<const f32x4 *>(st + 64 * c);
    const int64_t tok = (int64_t)heads * VEC;
    const float *src = packed + (int64_t)h * VEC;
    const float *knorm = packed + (int64_t)rows * tok + h;
    const float *vsrc = v + (int64_t)h * dim + min(16 * cb + (tid & 15), dim - 1);
    float *dst = out + (int64_t)h * dim + col;

    f32x4 ld[LOADS];
    float ldv = 0.0f, ldk = 0.0f;
    auto fetch = [&](int t0) {
#pragma unroll
        for (int i = 0; i < LOADS; i++) {
            const int x = tid + 256 * i, t = min(t0 + x / (VEC / 4), rows - 1);
            ld[i] = *reinterpret_cast<const f32x4 *>(src + t * tok + 4 * (x % (VEC / 4)));
        }
        if (tid < TB * 16) {
            const int64_t t = min(t0 + (tid >> 4), rows - 1);
            ldv = vsrc[t * v_stride];
            ldk = knorm[t * heads];
        }
    };
    auto stage = [&](float *to) {
#pragma unroll
        for (int i = 0; i < LOADS; i++) *reinterpret_cast<f32x4 *>(to + 4 * (tid + 256 * i)) = ld[i];
        if (tid < TB * 16) to[TB * VEC + tid] = ldv * ldk;
    };
    constexpr int BUF = TB * VEC + TB * 16;
    fetch(0);
    stage(smem);
    __syncthreads();
    int cur = 0;
    for (int t0 = 0; t0 < rows; t0 += TB) {
        const bool more = t0 + TB < rows;
        if (more) fetch(t0 + TB);
        const float *b = smem + cur * BUF, *bv = b + TB * VEC + 4 * wv + cg;
        const int n = min(TB, rows - t0);
        if (n == TB) {
            DeltaRows<NR> x[2];
            float vx[2], o[TB];
            x[0].load(b, sub);
            vx[0] = bv[0];
#pragma unroll
            for (int t = 0; t < TB; t++) {
                if (t + 1 < TB) {
                    x[(t + 1) & 1].load(b + (t + 1) * VEC, sub);
                    vx[(t + 1) & 1] = bv[16 * (t + 1)];
                }
                o[t] = delta_column<NR>(s, x[t & 1], vx[t & 1]);
            }
            // lane `sub` ends with the sum of token t0 + sub
            float mine = 0.0f;
#pragma unroll
            for (int t = 0; t < TB; t++) {
                const float sum = row16_sum(o[t]);
                mine = sub == t ? sum : mine;
            }
            if (sub < TB && col < dim) dst[(int64_t)(t0 + sub) * out_stride] = mine;
        } else {
            for (int t = 0; t < n; t++) {
                DeltaRows<NR> x;
                x.load(b + t * VEC, sub);
                const float o = row16_sum(delta_column<NR>(s, x, bv[16 * t]));
                if (sub == 0 && col < dim) dst[(int64_t)(t0 + t) * out_stride] = o;
            }
        }
        if (more) {
            stage(smem + (cur ^ 1) * BUF);
            __syncthreads();
            cur ^= 1;
        }
    }
    if (col < dim) {
#pragma unroll
        for (int c = 0; c < NR; c++) *reinterpret_cast<f32x4 *>(st + 64 * c) = s[c];
    }
}

struct DeltaStep {
    const float *row, *w0, *ab, *weight;
    const uint16_t *w2;
    float *state, *out;
    int64_t r_off, k_off, v_off, g_off, a_off, low_off, ldw2;
    int rank, heads, dim;
    float eps;
};

// One token, one head per workgroup of 16 waves.  The first 64 state columns are requested before anything else.
template <int NR>
__global__ __launch_bounds__(1024) void delta_step_kernel(DeltaStep a) {
    constexpr int SP = 64 * NR;
    extern __shared__ __attribute__((aligned(16))) float low[];           // tanh of the rank values, zero up to ldw2
    __shared__ __attribute__((aligned(16))) float vec[4 * SP], wl[SP], os[SP];
    __shared__ float s_inv, k_norm;
    const int tid = threadIdx.x, lane = tid & 63, wv = __builtin_amdgcn_readfirstlane(tid >> 6), sub = lane & 15, cg = lane >> 4;
    const int h = blockIdx.x;
    const int64_t hd = (int64_t)h * a.dim;
    f32x4 s[NR];
    float vj;
    auto load = [&](int c0) {
        const int col = min(c0 + cg, a.dim - 1);
        const float *st = a.state + (hd + col) * SP + 4 * sub;
#pragma unroll
        for (int c = 0; c < NR; c++) s[c] = *reinterpret_cast<const f32x4 *>(st + 64 * c);
        vj = a.row[a.v_off + hd + col];
    };
    load(4 * wv);
    for (int i = tid; i < a.ldw2; i += 1024) low[i] = i < a.rank ? tanhf(a.row[a.low_off + i]) : 0.0f;
    __syncthreads();
    for (int i0 = wv * 4; i0 < a.dim; i0 += 64) {
        const uint16_t *w = a.w2 + (hd + min(i0 + cg, a.dim - 1)) * a.ldw2;
        float acc = 0.0f;
        for (int j = 4 * sub; j < a.ldw2; j += 64) {
            const u32x2 x = *reinterpret_cast<const u32x2 *>(w + j);
            const f32x4 y = *reinterpret_cast<const f32x4 *>(low + j);
            acc = fmaf(__builtin_bit_cast(float, x.x << 16), y.x, acc);
            acc = fmaf(__builtin_bit_cast(float, x.x & 0xffff0000u), y.y, acc);
            acc = fmaf(__builtin_bit_cast(float, x.y << 16), y.z, acc);
            acc = fmaf(__builtin_bit_cast(float, x.y & 0xffff0000u), y.w, acc);
        }
        acc = row16_sum(acc);
        if (sub == 0 && i0 + cg < a.dim) wl[i0 + cg] = acc;
    }
    __syncthreads();
    if (wv == 0) {
        const float *x = a.row + hd;
        delta_pack(x + a.r_off, x + a.k_off, x + a.a_off, [&](int d) { return wl[d]; }, a.w0 + hd, a.ab + hd, vec, &k_norm, a.dim, SP, lane);
    }
    __syncthreads();
    DeltaRows<NR> x;
    x.load(vec, sub);
    for (int c0 = 4 * wv; c0 < a.dim; c0 += 64) {
        if (c0 >= 64) load(c0);
        const float o = row16_sum(delta_column<NR>(s, x, vj * k_norm));
        if (c0 + cg < a.dim) {
            float *st = a.state + (hd + c0 + cg) * SP + 4 * sub;
#pragma unroll
            for (int c = 0; c < NR; c++) *reinterpret_cast<f32x4 *>(st + 64 * c) = s[c];
            if (sub == 0) os[c0 + cg] = o;
        }
    }
    __syncthreads();
    if (wv == 0) {
        const float inv = head_inv_rms(os, a.dim, a.eps, lane);
        if (lane == 0) s_inv = inv;
    }
    __syncthreads();
    for (int e = tid; e < a.dim; e += 1024) a.out[hd + e] = os[e] * s_inv * a.weight[hd + e] * mix_sigmoid(a.row[a.g_off + hd + e]);
}

}  // namespace

extern "C" {

int64_t cq_mix_state_pad(int64_t dim) { return dim > 0 && dim <= CQ_MIX_MAX_DIM ? (dim <= 64 ? 64 : (dim <= 128 ? 128 : 256)) : -1; }

int64_t cq_mix_retention_workspace_bytes(int64_t rows, int64_t heads, int64_t dim, int64_t vdim) {
    if (rows <= 0 || heads <= 0 || dim <= 0 || vdim <= 0) return 0;
    int nseg, seg_len;
    retention_plan(rows, heads, vdim, &nseg, &seg_len);
    return nseg > 1 ? heads * ((vdim + 63) / 64) * nseg * ((dim + 15) / 16 * 16) * 64 * 4 : 0;
}

int cq_mix_retention(const float *q_dev, const float *k_dev, const float *v_dev, int64_t v_stride, const float *log2_decay_dev, float *state_dev,
                     float *out_dev, int64_t out_stride, int64_t rows, int64_t heads, int64_t dim, int64_t dim_pad, int64_t vdim, void *workspace_dev,
                     int64_t workspace_bytes, void *stream) {
    if (rows < 0 || heads <= 0 || dim <= 0 || vdim <= 0 || dim_pad != (dim + 15) / 16 * 16 || v_stride < heads * vdim || out_stride < heads * vdim)
        return CQ_ERR_SHAPE;
    if (rows == 0) return CQ_OK;
    if (!q_dev || !k_dev || !v_dev || !log2_decay_dev || !state_dev || !out_dev) return CQ_ERR_NULL;
    if (mix_misaligned(q_dev, 16) || mix_misaligned(k_dev, 16)) return CQ_ERR_ALIGN;
    if (dim > CQ_MIX_MAX_DIM || rows > (1 << 24) || heads * ((vdim + 63) / 64) > (1 << 20) || heads > 65535) return CQ_ERR_RANGE;
    Retention a;
    a.q = q_dev; a.k = k_dev; a.v = v_dev; a.log2_decay = log2_decay_dev;
    a.state = state_dev; a.out = out_dev; a.z = (float *)workspace_dev;
    a.v_stride = v_stride; a.out_stride = out_stride;
    a.rows = (int)rows; a.heads = (int)heads; a.dp = (int)dim_pad; a.vdim = (int)vdim; a.sp = (int)cq_mix_state_pad(dim);
    a.nvb = (a.vdim + 63) / 64;
    retention_plan(rows, heads, vdim, &a.nseg, &a.seg_len);
    if (a.nseg > 1 && (!workspace_dev || workspace_bytes < cq_mix_retention_workspace_bytes(rows, heads, dim, vdim))) return CQ_ERR_WORKSPACE;
    hipStream_t s = (hipStream_t)stream;
    const dim3 grid((unsigned)(a.heads * a.nvb), (unsigned)a.nseg);
    const size_t lds = (size_t)(a.dp + RC) * RLD * sizeof(float);
    if (lds > 64 * 1024) {
        const int e = (int)hipFuncSetAttribute(reinterpret_cast<const void *>(retention_kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e) return e;
    }
    if (a.nseg > 1) {
        hipLaunchKernelGGL(retention_segment_kernel, grid, dim3(256), 0, s, a);
        hipLaunchKernelGGL(retention_prefix_kernel, dim3((unsigned)((a.nvb * a.dp * 64 + 255) / 256), (unsigned)heads), dim3(256), 0, s, a);
    }
    hipLaunchKernelGGL(retention_kernel, grid, dim3(256), lds, s, a);
    return (int)hipGetLastError();
}

int cq_mix_talk_merge_retention_step(const void *workspace_dev, int64_t n_head, int64_t att_vdim, int64_t window, int64_t keep_first, int64_t ctx,
                                     float att_scale, float *att_out_dev, const float *row_dev, const cq_mix_heads *qk, int64_t v_off, int64_t g_off,
                                     const float *decay_dev, float *state_dev, int64_t heads, int64_t vdim, float eps, float ret_scale,
                                     float *ret_out_dev, const int32_t *pos_dev, int64_t pos, void *stream) {
    if (n_head <= 0 || att_vdim <= 0 || window < 1 || keep_first < 0 || ctx <= 0 || heads <= 0 || vdim <= 0 || v_off < 0 || g_off < 0 || pos < 0)
        return CQ_ERR_SHAPE;
    if (!workspace_dev || !att_out_dev || !row_dev || !qk || !decay_dev || !state_dev || !ret_out_dev) return CQ_ERR_NULL;
    for (int i = 0; i < 2; i++) {
        const int e = mix_check_group(qk[i], true);
        if (e) return e;
    }
    if (qk[0].heads != heads || qk[1].heads != heads || qk[0].dim != qk[1].dim) return CQ_ERR_SHAPE;
    if (mix_misaligned(state_dev, 16)) return CQ_ERR_ALIGN;
    if (qk[0].dim > CQ_MIX_MAX_DIM || vdim > 8192 || ctx > (1 << 28) || (!pos_dev && pos >= ctx)) return CQ_ERR_RANGE;
    StepArgs a;
    a.rec = (const float *)workspace_dev;
    a.n_head = (int)n_head; a.att_vdim = (int)att_vdim; a.ctx = (int)ctx;
    a.window = (int)(window < ctx ? window : ctx); a.keep_first = (int)(keep_first < ctx ? keep_first : ctx);
    const int64_t n_max = talk_max_keys(window, keep_first, ctx);
    a.splits = talk_splits(n_max); a.split_keys = talk_split_keys(n_max);
    a.att_scale = att_scale; a.ret_scale = ret_scale; a.eps = eps;
    a.att_out = att_out_dev; a.state = state_dev; a.ret_out = ret_out_dev; a.row = row_dev; a.decay = decay_dev;
    a.gq = qk[0]; a.gk = qk[1]; a.v_off = v_off; a.g_off = g_off; a.heads = (int)heads; a.vdim = (int)vdim;
    const int sp = (int)cq_mix_state_pad(qk[0].dim);
    const int f0 = (a.splits + 3) / 4 * 4 + 1024, f1 = 2 * sp + a.vdim;
    const size_t lds = (size_t)(f0 > f1 ? f0 : f1) * sizeof(float);
    if (lds > 64 * 1024) return CQ_ERR_RANGE;
    hipStream_t s = (hipStream_t)stream;
    const dim3 grid((unsigned)(n_head + heads));
    if (sp == 64) hipLaunchKernelGGL(talk_merge_retention_kernel<1>, grid, dim3(1024), lds, s, a, pos_dev, (int)pos);
    else if (sp == 128) hipLaunchKernelGGL(talk_merge_retention_kernel<2>, grid, dim3(1024), lds, s, a, pos_dev, (int)pos);
    else hipLaunchKernelGGL(talk_merge_retention_kernel<4>, grid, dim3(1024), lds, s, a, pos_dev, (int)pos);
    return (int)hipGetLastError();
}

int cq_mix_delta_prep(const float *row_dev, int64_t row_stride, int64_t r_off, int64_t k_off, int64_t a_off, const float *wl_dev, int64_t wl_stride,
                      const float *w0_dev, const float *a_bias_dev, float *packed_dev, int64_t rows, int64_t heads, int64_t dim, void *stream) {
    if (rows < 0 || heads <= 0 || dim <= 0 || r_off < 0 || k_off < 0 || a_off < 0 || wl_stride < heads * dim) return CQ_ERR_SHAPE;
    const int64_t top = (r_off > k_off ? r_off : k_off) > a_off ? (r_off > k_off ? r_off : k_off) : a_off;
    if (row_stride < top + heads * dim) return CQ_ERR_SHAPE;
    if (rows == 0) return CQ_OK;
    if (!row_dev || !wl_dev || !w0_dev || !a_bias_dev || !packed_dev) return CQ_ERR_NULL;
    if (dim > CQ_MIX_MAX_DIM || heads > 4 * 65535 || rows > 0x7fffffffLL) return CQ_ERR_RANGE;
    hipLaunchKernelGGL(delta_prep_kernel, dim3((unsigned)rows, (unsigned)((heads + 3) / 4)), dim3(256), 0, (hipStream_t)stream, row_dev, row_stride, r_off, k_off, a_off,
                       wl_dev, wl_stride, w0_dev, a_bias_dev, packed_dev, rows, (int)heads, (int)dim, (int)cq_mix_state_pad(dim));
    return (int)hipGetLastError();
}

int cq_mix_delta_scan(const float *packed_dev, const float *v_dev, int64_t v_stride, float *state_dev, float *out_dev, int64_t out_stride, int64_t rows,
                      int64_t heads, int64_t dim, void *stream) {
    if (rows < 0 || heads <= 0 || dim <= 0 || v_stride < heads * dim || out_stride < heads * dim) return CQ_ERR_SHAPE;
    if (rows == 0) return CQ_OK;
    if (!packed_dev || !v_dev || !state_dev || !out_dev) return CQ_ERR_NULL;
    if (mix_misaligned(packed_dev, 16) || mix_misaligned(state_dev, 16)) return CQ_ERR_ALIGN;
    if (dim > CQ_MIX_MAX_DIM || heads > (1 << 20) || rows > (1 << 24)) return CQ_ERR_RANGE;
    const int ncb = (int)((dim + 15) / 16), sp = (int)cq_mix_state_pad(dim);
    const dim3 grid((unsigned)((heads + 7) / 8 * 8 * ncb));
    hipStream_t s = (hipStream_t)stream;
#define CQ_DS(NR_, TB_)                                                                                                                                   \
    do {                                                                                                                                                   \
        const size_t lds = (size_t)2 * (TB_ * 4 * 64 * NR_ + TB_ * 16) * sizeof(float);                                                                    \
        if (lds > 64 * 1024) {                                                                                                                             \
            const int e = (int)hipFuncSetAttribute(reinterpret_cast<const void *>(delta_scan_kernel<NR_, TB_>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds); \
            if (e) return e;                                                                                                                               \
        }                                                                                                                                                  \
        hipLaunchKernelGGL((delta_scan_kernel<NR_, TB_>), grid, dim3(256), lds, s, packed_dev, v_dev, v_stride, state_dev, out_dev, out_stride, (int)rows,  \
                           (int)heads, (int)dim, ncb);                                                                                                     \
    } while (0)
    if (sp == 64) CQ_DS(1, 16);
    else if (sp == 128) CQ_DS(2, 8);
    else CQ_DS(4, 8);
#undef CQ_DS
    return (int)hipGetLastError();
}

int cq_mix_delta_step(const float *row_dev, int64_t r_off, int64_t k_off, int64_t v_off, int64_t g_off, int64_t a_off, int64_t low_off, const void *w2_dev,
                      int64_t ldw2, int64_t rank, const float *w0_dev, const float *a_bias_dev, const float *weight_dev, float *state_dev, float *out_dev,
                      int64_t heads, int64_t dim, float eps, void *stream) {
    if (heads <= 0 || dim <= 0 || rank <= 0 || ldw2 < rank || ldw2 % 64 || r_off < 0 || k_off < 0 || v_off < 0 || g_off < 0 || a_off < 0 || low_off < 0)
        return CQ_ERR_SHAPE;
    if (!row_dev || !w2_dev || !w0_dev || !a_bias_dev || !weight_dev || !state_dev || !out_dev) return CQ_ERR_NULL;
    if (mix_misaligned(w2_dev, 16) || mix_misaligned(state_dev, 16)) return CQ_ERR_ALIGN;
    if (dim > CQ_MIX_MAX_DIM || heads > (1 << 20) || ldw2 > 8192) return CQ_ERR_RANGE;
    DeltaStep a;
    a.row = row_dev; a.w0 = w0_dev; a.ab = a_bias_dev; a.weight = weight_dev; a.w2 = (const uint16_t *)w2_dev; a.state = state_dev; a.out = out_dev;
    a.r_off = r_off; a.k_off = k_off; a.v_off = v_off; a.g_off = g_off; a.a_off = a_off; a.low_off = low_off; a.ldw2 = ldw2;
    a.rank = (int)rank; a.heads = (int)heads; a.dim = (int)dim; a.eps = eps;
    const size_t lds = (size_t)ldw2 * sizeof(float);
    hipStream_t s = (hipStream_t)stream;
    const int sp = (int)cq_mix_state_pad(dim);
    if (sp == 64) hipLaunchKernelGGL(delta_step_kernel<1>, dim3((unsigned)heads), dim3(1024), lds, s, a);
    else if (sp == 128) hipLaunchKernelGGL(delta_step_kernel<2>, dim3((unsigned)heads), dim3(1024), lds, s, a);
    else hipLaunchKernelGGL(delta_step_kernel<4>, dim3((unsigned)heads), dim3(1024), lds, s, a);
    return (int)hipGetLastError();
}

}  // extern "C"
