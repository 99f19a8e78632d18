// Attention whose keys and values are cached per group of query heads, with a sliding window.
//
// Queries and keys are normed over all their rows at once, or head by head; a workgroup prepares a whole token: sums of squares, the norms'
// weights, the rotation, and the cache write.  The attention kernels work on rows that are (token, query head) pairs of one sequence and
// key / value head: G = heads / kv_heads rows of a token share every key they read.
//
// Scores are taken transposed, Sᵀ = K·Qᵀ, so that a row's statistics stay in one column of lanes and P leaves the accumulators as the
// operand of Oᵀ += Vᵀ·Pᵀ without a detour: the contraction index (lane group a, j < 4) is key 4a + j of one 16-key block, (a, j ≥ 4)
// key 4a + j − 4 of the next, and the value cache is laid out to match.
#include <math.h>

#include <algorithm>

#include "common.h"
#include "grouped_cache.h"
#include "knobs.h"
#include "layer_ops.h"
#include "seq_tiles.h"

namespace fh {

// one workgroup per token
template <typename E>
__global__ __launch_bounds__(256) void grouped_prepare_kernel(GroupedDims d, GroupedBuffers<E> p, BatchView v) {
    typedef typename Frag<E>::v8 v8;
    __shared__ float red[8];
    const int t = blockIdx.x, tid = threadIdx.x, seq = v.tok_seq[t];
    const long pos = (long)v.pos[seq] + t - v.cu[seq];
    const int nq = d.heads * d.dp, nk = d.kv_heads * d.dp, nv = d.kv_heads * d.vp;
    const E *qr = p.q_in + t * p.ld, *kr = p.k_in + t * p.ld, *vr = p.v_in + t * p.ld;
    float sq = 0.f, sk = 0.f;
    for (int i = tid * 8; i < nq + nk; i += 2048) {
        const v8 x = *reinterpret_cast<const v8*>(i < nq ? qr + i : kr + (i - nq));
        float s = 0.f;
#pragma unroll
        for (int j = 0; j < 8; j++) s += (float)x[j] * (float)x[j];           // (padded columns are zero)
        if (i < nq) sq += s; else sk += s;
    }
    sq = wave_reduce_sum(sq);
    sk = wave_reduce_sum(sk);
    if ((tid & 63) == 0) { red[tid >> 6] = sq; red[4 + (tid >> 6)] = sk; }
    const long block = v.bt[(long)seq * v.max_blocks + pos / 16];
    const int slot = pos % 16;
    __syncthreads();
    const float iq = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)(d.heads * d.dim) + p.eps);
    const float ik = 1.0f / sqrtf((red[4] + red[5] + red[6] + red[7]) / (float)(d.kv_heads * d.dim) + p.eps);
    for (int i = tid * 8; i < nq + nk; i += 2048) {
        const bool query = i < nq;
        const int c = query ? i : i - nq, dim0 = c % d.dp;
        const v8 x = *reinterpret_cast<const v8*>((query ? qr : kr) + c);
        const float *w = (query ? p.q_norm : p.k_norm) + c, inv = query ? iq : ik;
        floatx8 f;
#pragma unroll
        for (int j = 0; j < 8; j++) f[j] = (float)x[j] * inv * w[j];
        f = rot_apply(f, rot_load(dim0, d.rot_dims, p.cos_t, p.sin_t, pos));
        v8 o;
#pragma unroll
        for (int j = 0; j < 8; j++) o[j] = (E)f[j];
        E* dst = query ? p.q + (long)t * nq + c : p.k_pool + (block * d.kv_heads + c / d.dp) * d.dp * 16 + (dim0 * 2 + slot) * 8;
        *reinterpret_cast<v8*>(dst) = o;
    }
    E* vt = p.v_pool + block * d.kv_heads * d.vp * 16;
    for (int i = tid; i < nv; i += 256) vt[(long)(i / d.vp) * d.vp * 16 + value_offset(slot, i % d.vp)] = vr[i];
}

// the same with norms of one head each: a power of two of lanes (`sub`) per head, 8 dimensions a lane
template <typename E>
__global__ __launch_bounds__(256) void grouped_prepare_heads_kernel(GroupedDims d, GroupedBuffers<E> p, BatchView v, int sub) {
    typedef typename Frag<E>::v8 v8;
    const int t = blockIdx.x, tid = threadIdx.x, seq = v.tok_seq[t], lane = tid & (sub - 1);
    const long pos = (long)v.pos[seq] + t - v.cu[seq];
    const long block = v.bt[(long)seq * v.max_blocks + pos / 16];
    const int slot = pos % 16, nk = p.k_in ? d.kv_heads : 0;
    for (int h = tid / sub; h < d.heads + nk; h += 256 / sub) {
        const bool query = h < d.heads;
        const int kh = h - d.heads;
        const E* src = query ? p.q_in + t * p.ld + (long)h * d.dp : p.k_in + t * p.ld + (long)kh * d.dp;
        const float* w = query ? p.q_norm : p.k_norm;
        float s = 0.f;
        for (int i = lane * 8; i < d.dp; i += sub * 8) {
            const v8 x = *reinterpret_cast<const v8*>(src + i);
#pragma unroll
            for (int j = 0; j < 8; j++) s += (float)x[j] * (float)x[j];       // (padded columns are zero)
        }
        for (int off = 1; off < sub; off <<= 1) s += __shfl_xor(s, off, 64);
        const float inv = 1.0f / sqrtf(s / (float)d.dim + p.eps);
        for (int i = lane * 8; i < d.dp; i += sub * 8) {
            const v8 x = *reinterpret_cast<const v8*>(src + i);
            floatx8 f;
#pragma unroll
            for (int j = 0; j < 8; j++) f[j] = (float)x[j] * inv * w[i + j];
            f = rot_apply(f, rot_load(i, d.rot_dims, p.cos_t, p.sin_t, pos));
            v8 o;
#pragma unroll
            for (int j = 0; j < 8; j++) o[j] = (E)f[j];
            E* dst = query ? p.q + ((long)t * d.heads + h) * d.dp + i : p.k_pool + (block * d.kv_heads + kh) * d.dp * 16 + (i * 2 + slot) * 8;
            *reinterpret_cast<v8*>(dst) = o;
        }
    }
    if (!p.k_in) return;
    const E* vr = p.v_in + t * p.ld;
    E* vt = p.v_pool + block * d.kv_heads * d.vp * 16;
    for (int i = tid; i < d.kv_heads * d.vp; i += 256) vt[(long)(i / d.vp) * d.vp * 16 + value_offset(slot, i % d.vp)] = vr[i];
}

// factor of a row's Σ e^(score − m)·value (l: with the sink)
template <typename E>
__device__ __forceinline__ float grouped_factor(const GroupedBuffers<E>& p, float l, long tok, int head) {
    float f = l > 0.f ? p.mult / l : 0.f;
    if (p.gate) f *= (float)p.gate[tok * p.ld_gate + head];
    return f;
}

// ── plain form: one workgroup per (token, head), 256 keys at a time; any size, both number formats ──
template <typename E>
__global__ __launch_bounds__(256) void grouped_attn_plain_kernel(GroupedDims d, GroupedBuffers<E> p, BatchView v) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, wave = tid >> 6, kvh = h / (d.heads / d.kv_heads);
    float *q = lds, *pr = lds + d.dp, *red = pr + 256, *o = red + 8;          // [dp] query, [256] weights, [8], [vp] output
    const int seq = v.tok_seq[t], pos = v.pos[seq] + t - v.cu[seq];
    for (int i = tid; i < d.dp; i += 256) q[i] = (float)p.q[((long)t * d.heads + h) * d.dp + i];
    for (int i = tid; i < d.vp; i += 256) o[i] = 0.f;
    const int lo = max(0, pos + 1 - d.window), hi = pos + 1;
    const int32_t* bt = v.bt + (long)seq * v.max_blocks;
    float m_run = -INFINITY, l_run = 0.f;
    __syncthreads();
    for (int k0 = lo; k0 < hi; k0 += 256) {
        const int key = k0 + tid;
        float sc = -INFINITY;
        if (key < hi) {
            const E* kt = p.k_pool + ((long)bt[key / 16] * d.kv_heads + kvh) * d.dp * 16 + (key % 16) * 8;
            float acc = 0.f;
            for (int i = 0; i < d.dp; i += 8) {
                const typename Frag<E>::v8 x = *reinterpret_cast<const typename Frag<E>::v8*>(kt + i * 16);
#pragma unroll
                for (int j = 0; j < 8; j++) acc += q[i + j] * (float)x[j];
            }
            sc = acc * d.scale;
            if (p.r1) sc -= p.r1[h] * log1pf(p.r2[h] * (float)(pos - key));
        }
        const float mx = wave_reduce_max(sc);
        if ((tid & 63) == 0) red[wave] = mx;
        __syncthreads();
        const float m_new = fmaxf(fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])), m_run);
        const float pv = expf(sc - m_new), alpha = expf(m_run - m_new);       // (key lo is visible: m_new is finite)
        pr[tid] = pv;
        const float ps = wave_reduce_sum(pv);
        if ((tid & 63) == 0) red[4 + wave] = ps;
        __syncthreads();
        l_run = l_run * alpha + red[4] + red[5] + red[6] + red[7];
        m_run = m_new;
        const int n = min(256, hi - k0);
        for (int i = tid; i < d.vp; i += 256) {
            float acc = o[i] * alpha;
            for (int k = 0; k < n; k++) {
                const int kk = k0 + k;
                acc += pr[k] * (float)p.v_pool[((long)bt[kk / 16] * d.kv_heads + kvh) * d.vp * 16 + value_offset(kk % 16, i)];
            }
            o[i] = acc;
        }
        __syncthreads();
    }
    if (p.sink) l_run += expf(p.sink[h] - m_run);
    const float f = grouped_factor(p, l_run, t, h);
    for (int i = tid; i < d.vp; i += 256) {
        const float g = p.value_gate ? (float)p.value_gate[t * p.ld_value_gate + h * d.vp + i] : 1.f;
        p.out[(long)t * p.ldo + h * d.vp + i] = (E)(o[i] * f * g);
    }
}

// ── matrix-core forms; DS: 32-wide steps of a head (dp = vp) ──
constexpr int GROUPED_PARTIAL_PAD = 4;       // floats behind a partial row's outputs: maximum, sum
typedef short shortx8 __attribute__((ext_vector_type(8)));
// four elements of a row's result: columns [col, col + 4) of the concatenated heads
__device__ __forceinline__ void grouped_store4(const GroupedBuffers<bf16>& p, long tok, int col, floatx4 x, float f) {
    bf16x4 y;
    if (p.value_gate) {
        const bf16x4 g = *reinterpret_cast<const bf16x4*>(p.value_gate + tok * p.ld_value_gate + col);
#pragma unroll
        for (int r = 0; r < 4; r++) y[r] = (bf16)(x[r] * f * (float)g[r]);
    } else {
#pragma unroll
        for (int r = 0; r < 4; r++) y[r] = (bf16)(x[r] * f);
    }
    *reinterpret_cast<bf16x4*>(p.out + tok * p.ldo + col) = y;
}

// Few rows per sequence.  grid (16-row tiles × KV splits, kv_heads): the four waves take 32-key steps of the range in turn, straight from
// the cache into registers (the next step is requested before this one is used), and merge through LDS.
// FAR: scores fall with the logarithm of the distance.
template <int DS, bool FAR>
__global__ __launch_bounds__(256) void grouped_attn_keys_kernel(GroupedDims d, GroupedBuffers<bf16> p, BatchView v, int nsplit) {
    constexpr int DT = 2 * DS, D = 32 * DS, LD = D + 4;
    extern __shared__ __attribute__((aligned(16))) float lds_o[];              // [4][16][LD]
    __shared__ float lds_m[64], lds_l[64];
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63, a = lane >> 4, b = lane & 15;
    const int split = blockIdx.x % nsplit, tile_id = blockIdx.x / nsplit, kvh = blockIdx.y, G = d.heads / d.kv_heads;
    SeqTile w;
    if (!find_seq_tile(v, G, 16, tile_id, &w)) return;
    const int rows = w.q_len * G, rho = w.tile * 16 + b;
    const bool ok = rho < rows;
    const int tl = ok ? rho / G : 0, head = kvh * G + (ok ? rho - tl * G : 0), row_pos = w.pos0 + tl, win_lo = max(0, row_pos + 1 - d.window);
    const long tok = w.tok0 + tl;
    const float r1 = FAR ? p.r1[head] : 0.f, r2 = FAR ? p.r2[head] : 0.f;
    const int t_first = w.tile * 16 / G, t_last = min(w.q_len - 1, (w.tile * 16 + 15) / G);
    const int blk_lo = max(0, w.pos0 + t_first + 1 - d.window) / 16, blk_hi = (w.pos0 + t_last + 16) / 16, nstep = (blk_hi - blk_lo + 1) / 2;
    const int st_lo = nstep * split / nsplit, st_hi = nstep * (split + 1) / nsplit;
    const int32_t* bt = v.bt + (long)w.seq * v.max_blocks;
    bf16x8 qf[DS], kf[2][2][DS], vf[2][2][DS];
    const long kd = (long)d.kv_heads * D * 16, off = (long)kvh * D * 16 + lane * 8;
    auto load = [&](int buf, int st) {                                         // (past the end: a copy of the last block, masked below)
#pragma unroll
        for (int i = 0; i < 2; i++) {
            const long blk = __builtin_amdgcn_readfirstlane(bt[min(blk_lo + 2 * st + i, blk_hi - 1)]);
#pragma unroll
            for (int s = 0; s < DS; s++) {
                kf[buf][i][s] = *reinterpret_cast<const bf16x8*>(p.k_pool + blk * kd + off + s * 512);
                vf[buf][i][s] = *reinterpret_cast<const bf16x8*>(p.v_pool + blk * kd + off + s * 512);
            }
        }
    };
#pragma unroll
    for (int s = 0; s < DS; s++) qf[s] = *reinterpret_cast<const bf16x8*>(p.q + (tok * d.heads + head) * D + 32 * s + 8 * a);
    float m_run = -INFINITY, l_run = 0.f;
    floatx4 o[DT];
#pragma unroll
    for (int t = 0; t < DT; t++) o[t] = (floatx4){0.f, 0.f, 0.f, 0.f};
    auto step = [&](int buf, int st) {
        float sc[8], mx = -INFINITY;
#pragma unroll
        for (int i = 0; i < 2; i++) {
            floatx4 s2[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
            for (int s = 0; s < DS; s++) s2[s & 1] = Frag<bf16>::mma(kf[buf][i][s], qf[s], s2[s & 1]);
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const int key = (blk_lo + 2 * st + i) * 16 + 4 * a + r;
                float z = (s2[0][r] + s2[1][r]) * d.scale;
                if (FAR) z -= r1 * __logf(1.0f + r2 * (float)max(row_pos - key, 0));
                sc[4 * i + r] = ok && key <= row_pos && key >= win_lo ? z : -INFINITY;
                mx = fmaxf(mx, sc[4 * i + r]);
            }
        }
        const float m_new = fmaxf(m_run, rows_reduce_max(mx)), m_safe = m_new == -INFINITY ? 0.f : m_new, alpha = __expf(m_run - m_safe);
        bf16x8 pf;
        float ps = 0.f;
#pragma unroll
        for (int j = 0; j < 8; j++) { const float e = __expf(sc[j] - m_safe); ps += e; pf[j] = (bf16)e; }
        l_run = l_run * alpha + ps;                                            // (this lane's keys; the four lane groups meet at the end)
        m_run = m_new;
#pragma unroll
        for (int t = 0; t < DT; t++) {
#pragma unroll
            for (int r = 0; r < 4; r++) o[t][r] *= alpha;
            o[t] = Frag<bf16>::mma(value_operand(vf[buf][0][t >> 1], vf[buf][1][t >> 1], t & 1), pf, o[t]);
        }
    };
    if (st_lo + wave < st_hi) {
        int st = st_lo + wave;
        load(0, st);
        while (true) {
            load(1, st + 4);
            step(0, st);
            st += 4;
            if (st >= st_hi) break;
            load(0, st + 4);
            step(1, st);
            st += 4;
            if (st >= st_hi) break;
        }
    }
    const float l_own = rows_reduce_sum(l_run);
    if (a == 0) { lds_m[wave * 16 + b] = m_run; lds_l[wave * 16 + b] = l_own; }
    __syncthreads();
    float M = -INFINITY, L = 0.f;
#pragma unroll
    for (int i = 0; i < 4; i++) M = fmaxf(M, lds_m[i * 16 + b]);
    const float M_safe = M == -INFINITY ? 0.f : M;
#pragma unroll
    for (int i = 0; i < 4; i++) L += lds_l[i * 16 + b] * __expf(lds_m[i * 16 + b] - M_safe);
    const float f_own = __expf(m_run - M_safe);
#pragma unroll
    for (int t = 0; t < DT; t++) {
        floatx4 x;
#pragma unroll
        for (int r = 0; r < 4; r++) x[r] = o[t][r] * f_own;
        *reinterpret_cast<floatx4*>(lds_o + (wave * 16 + b) * LD + t * 16 + 4 * a) = x;
    }
    __syncthreads();
    if (a == 0 && wave == 0) { lds_m[b] = M; lds_l[b] = L; }
    __syncthreads();
    for (int i = threadIdx.x; i < 16 * (D / 4); i += 256) {
        const int row = i / (D / 4), c = (i % (D / 4)) * 4, ro = w.tile * 16 + row;
        if (ro >= rows) continue;
        floatx4 x = *reinterpret_cast<const floatx4*>(lds_o + row * LD + c);
#pragma unroll
        for (int q = 1; q < 4; q++) x += *reinterpret_cast<const floatx4*>(lds_o + (q * 16 + row) * LD + c);
        if (nsplit > 1) {
            float* dst = p.partial + (((long)blockIdx.y * gridDim.x + blockIdx.x) * 16 + row) * (D + GROUPED_PARTIAL_PAD);
            *reinterpret_cast<floatx4*>(dst + c) = x;
            if (c == 0) { dst[D] = lds_m[row]; dst[D + 1] = lds_l[row]; }
            continue;
        }
        const int rt = ro / G, rh = kvh * G + ro % G;
        const float sink = p.sink ? __expf(p.sink[rh] - lds_m[row]) : 0.f;
        grouped_store4(p, w.tok0 + rt, rh * D + c, x, grouped_factor(p, lds_l[row] + sink, w.tok0 + rt, rh));
    }
}
// grid (tiles, kv_heads): one thread per (row, 4 dimensions)
__global__ __launch_bounds__(256) void grouped_attn_reduce_kernel(GroupedDims d, GroupedBuffers<bf16> p, BatchView v, int nsplit) {
    const int G = d.heads / d.kv_heads, kvh = blockIdx.y, quads = d.vp / 4;
    SeqTile w;
    if (!find_seq_tile(v, G, 16, blockIdx.x, &w)) return;
    for (int i = threadIdx.x; i < 16 * quads; i += 256) {
        const int row = i / quads, c = (i % quads) * 4, ro = w.tile * 16 + row;
        if (ro >= w.q_len * G) continue;
        const long ld = d.vp + GROUPED_PARTIAL_PAD;
        const float* src = p.partial + (((long)kvh * gridDim.x + blockIdx.x) * nsplit * 16 + row) * ld;
        float M = -INFINITY, L = 0.f;
        for (int z = 0; z < nsplit; z++) M = fmaxf(M, src[z * 16 * ld + d.vp]);
        floatx4 acc = {0.f, 0.f, 0.f, 0.f};
        for (int z = 0; z < nsplit; z++) {
            const float f = __expf(src[z * 16 * ld + d.vp] - M);
            L += src[z * 16 * ld + d.vp + 1] * f;
            acc += *reinterpret_cast<const floatx4*>(src + z * 16 * ld + c) * f;
        }
        const int rt = ro / G, rh = kvh * G + ro % G;
        if (p.sink) L += __expf(p.sink[rh] - M);
        grouped_store4(p, w.tok0 + rt, rh * d.vp + c, acc, grouped_factor(p, L, w.tok0 + rt, rh));
    }
}

// Prompts.  grid (128-row tiles, kv_heads): 4 waves × 2 tiles of 16 rows.  64 keys per step: wave w copies block w of the step's keys and
// values into LDS with the load unit, double-buffered.
template <int DS, bool FAR>
__global__ __launch_bounds__(256, DS <= 4 ? 2 : 1) void grouped_attn_tile_kernel(GroupedDims d, GroupedBuffers<bf16> p, BatchView v) {
    constexpr int MT = 2, DT = 2 * DS, D = 32 * DS, BLK = 2 * DS * 512;
    extern __shared__ __attribute__((aligned(16))) bf16 lds_x[];               // [2][4 blocks][BLK]: keys, values
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63, a = lane >> 4, b = lane & 15;
    const int kvh = blockIdx.y, G = d.heads / d.kv_heads;
    SeqTile w;
    if (!find_seq_tile_last_first(v, G, 128, blockIdx.x, &w)) return;
    const int rows = w.q_len * G;
    const float sl2 = d.scale * 1.4426950408889634f;
    bf16x8 qf[MT][DS];
    int row_pos[MT], win_lo[MT], vis_lo[MT], vis_hi[MT], head[MT];
    long tok[MT];
    bool ok[MT];
    float r1[MT], r2[MT];
#pragma unroll
    for (int mt = 0; mt < MT; mt++) {
        const int r0 = w.tile * 128 + (wave * MT + mt) * 16, rho = min(r0 + b, rows - 1), tl = rho / G;
        ok[mt] = r0 + b < rows;
        head[mt] = kvh * G + rho - tl * G;
        tok[mt] = w.tok0 + tl;
        if (FAR) { r1[mt] = p.r1[head[mt]]; r2[mt] = p.r2[head[mt]]; }
        row_pos[mt] = w.pos0 + tl;
        win_lo[mt] = max(0, row_pos[mt] + 1 - d.window);
        vis_hi[mt] = r0 + 15 < rows ? w.pos0 + r0 / G : -1;                    // keys in [vis_lo, vis_hi] are seen by every row of the tile
        vis_lo[mt] = max(0, w.pos0 + (r0 + 15) / G + 1 - d.window);
        const bf16* q = p.q + (tok[mt] * d.heads + head[mt]) * D + 8 * a;
#pragma unroll
        for (int s = 0; s < DS; s++) qf[mt][s] = *reinterpret_cast<const bf16x8*>(q + 32 * s);
    }
    const int t_first = w.tile * 128 / G, t_last = min(w.q_len - 1, (w.tile * 128 + 127) / G);
    const int blk_lo = max(0, w.pos0 + t_first + 1 - d.window) / 16, blk_hi = (w.pos0 + t_last + 16) / 16, nstep = (blk_hi - blk_lo + 3) / 4;
    const int32_t* bt = v.bt + (long)w.seq * v.max_blocks;
    const long kd = (long)d.kv_heads * D * 16, off = (long)kvh * D * 16 + lane * 8;
    auto issue = [&](long blk, int buf) {
        bf16* dst = lds_x + (buf * 4 + wave) * BLK;
#define GA_COPY(src, slot) __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(src), (__attribute__((address_space(3))) void*)(dst + (slot) * 512), 16, 0, 0)
#pragma unroll
        for (int s = 0; s < DS; s++) GA_COPY(p.k_pool + blk * kd + off + s * 512, s);
#pragma unroll
        for (int s = 0; s < DS; s++) GA_COPY(p.v_pool + blk * kd + off + s * 512, DS + s);
#undef GA_COPY
    };
    auto block_of = [&](int st) { return (long)__builtin_amdgcn_readfirstlane(bt[min(blk_lo + 4 * st + wave, blk_hi - 1)]); };      // (past the end: a copy of the last, masked)
    float m_run[MT], l_run[MT];
    floatx4 o[MT][DT];
#pragma unroll
    for (int mt = 0; mt < MT; mt++) {
        m_run[mt] = -INFINITY; l_run[mt] = 0.f;
#pragma unroll
        for (int t = 0; t < DT; t++) o[mt][t] = (floatx4){0.f, 0.f, 0.f, 0.f};
    }
    issue(block_of(0), 0);
    long next = block_of(1);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    for (int st = 0; st < nstep; st++) {
        const int buf = st & 1;
        if (st + 1 < nstep) { issue(next, buf ^ 1); next = block_of(st + 2); }
        const bf16* kb = lds_x + buf * 4 * BLK + lane * 8;
        floatx4 sv[MT][4];
#pragma unroll
        for (int mt = 0; mt < MT; mt++)
#pragma unroll
            for (int i = 0; i < 4; i++) sv[mt][i] = (floatx4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < DS; s++)
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const bf16x8 k = *reinterpret_cast<const bf16x8*>(kb + i * BLK + s * 512);
#pragma unroll
                for (int mt = 0; mt < MT; mt++) sv[mt][i] = Frag<bf16>::mma(k, qf[mt][s], sv[mt][i]);
            }
        bf16x8 pf[MT][2];
        const int key0 = (blk_lo + 4 * st) * 16;
#pragma unroll
        for (int mt = 0; mt < MT; mt++) {
            if (FAR) {                                                         // scores in base 2 from here
                const int d0 = row_pos[mt] - key0 - 4 * a;
#pragma unroll
                for (int i = 0; i < 4; i++)
#pragma unroll
                    for (int r = 0; r < 4; r++)
                        sv[mt][i][r] = __builtin_fmaf(sv[mt][i][r], sl2, -r1[mt] * __builtin_amdgcn_logf(__builtin_fmaf(r2[mt], (float)max(d0 - i * 16 - r, 0), 1.0f)));
            }
            if (!(key0 + 63 <= vis_hi[mt] && key0 >= vis_lo[mt])) {
#pragma unroll
                for (int i = 0; i < 4; i++)
#pragma unroll
                    for (int r = 0; r < 4; r++) {
                        const int key = key0 + i * 16 + 4 * a + r;
                        if (!(ok[mt] && key <= row_pos[mt] && key >= win_lo[mt])) sv[mt][i][r] = -INFINITY;
                    }
            }
            float mx = -INFINITY;
#pragma unroll
            for (int i = 0; i < 4; i++) mx = fmaxf(mx, fmaxf(fmaxf(sv[mt][i][0], sv[mt][i][1]), fmaxf(sv[mt][i][2], sv[mt][i][3])));
            mx = rows_reduce_max(FAR ? mx : mx * sl2);                                    // (scale > 0, checked by the caller: the maximum commutes)
            const float m_new = fmaxf(m_run[mt], mx), m_safe = m_new == -INFINITY ? 0.f : m_new;
            if (__ballot(m_new != m_run[mt]) != 0) {
                const float alpha = __builtin_amdgcn_exp2f(m_run[mt] - m_safe);
#pragma unroll
                for (int t = 0; t < DT; t++)
#pragma unroll
                    for (int r = 0; r < 4; r++) o[mt][t][r] *= alpha;
                l_run[mt] *= alpha;
                m_run[mt] = m_new;
            }
#pragma unroll
            for (int i = 0; i < 4; i++)
#pragma unroll
                for (int r = 0; r < 4; r++) {
                    const float e = __builtin_amdgcn_exp2f(FAR ? sv[mt][i][r] - m_safe : __builtin_fmaf(sv[mt][i][r], sl2, -m_safe));
                    l_run[mt] += e;
                    pf[mt][i >> 1][(i & 1) * 4 + r] = (bf16)e;
                }
        }
#pragma unroll
        for (int c = 0; c < 2; c++) {
            const bf16* vb = kb + 2 * c * BLK + DS * 512;
#pragma unroll
            for (int s = 0; s < DS; s++) {
                const bf16x8 v0 = *reinterpret_cast<const bf16x8*>(vb + s * 512), v1 = *reinterpret_cast<const bf16x8*>(vb + BLK + s * 512);
#pragma unroll
                for (int sub = 0; sub < 2; sub++)
#pragma unroll
                    for (int mt = 0; mt < MT; mt++) o[mt][2 * s + sub] = Frag<bf16>::mma(value_operand(v0, v1, sub), pf[mt][c], o[mt][2 * s + sub]);
            }
        }
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();
    }
#pragma unroll
    for (int mt = 0; mt < MT; mt++) {
        float l = rows_reduce_sum(l_run[mt]);
        if (!ok[mt]) continue;
        if (p.sink) l += __builtin_amdgcn_exp2f(p.sink[head[mt]] * 1.4426950408889634f - m_run[mt]);
        const float f = grouped_factor(p, l, tok[mt], head[mt]);
#pragma unroll
        for (int t = 0; t < DT; t++) grouped_store4(p, tok[mt], head[mt] * D + 4 * a + t * 16, o[mt][t], f);
    }
}

template <typename E>
int grouped_prepare(const GroupedDims& d, const GroupedBuffers<E>& b, const BatchView& v, hipStream_t s) {
    FH_REQUIRE(b.k_in || b.head_norm, "grouped attention: keys and values of another layer take norms of one head each");
    int sub = 1;
    while (sub < 64 && sub * 8 < d.dp) sub *= 2;
    if (b.head_norm) hipLaunchKernelGGL(grouped_prepare_heads_kernel<E>, dim3(v.T), dim3(256), 0, s, d, b, v, sub);
    else hipLaunchKernelGGL(grouped_prepare_kernel<E>, dim3(v.T), dim3(256), 0, s, d, b, v);
    FH_CHECK_LAUNCH();
    return 0;
}

template <typename E>
static int grouped_plain(const GroupedDims& d, const GroupedBuffers<E>& b, const BatchView& v, hipStream_t s) {
    form_hit(FORM_GROUPED_ATTN_PLAIN);
    const size_t lds = (size_t)(d.dp + d.vp + 256 + 8) * 4;
    FH_REQUIRE(lds <= 64 * 1024, "grouped attention: heads of %d / %d do not fit LDS", d.dim, d.vdim);
    hipLaunchKernelGGL(grouped_attn_plain_kernel<E>, dim3(v.T, d.heads), dim3(256), lds, s, d, b, v);
    FH_CHECK_LAUNCH();
    return 0;
}
template <int DS, bool FAR>
static int grouped_tile(const GroupedDims& d, const GroupedBuffers<bf16>& b, const BatchView& v, hipStream_t s) {
    constexpr size_t lds = (size_t)2 * 4 * 2 * DS * 1024;
    static bool attr = false;
    if (!attr) { FH_CHECK_HIP(hipFuncSetAttribute((const void*)grouped_attn_tile_kernel<DS, FAR>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds)); attr = true; }
    const int tiles = (int)((long)v.T * (d.heads / d.kv_heads) / 128) + v.num_seqs;      // upper bound of Σ ceil(rows of a sequence / 128)
    form_hit(FORM_GROUPED_ATTN_TILE);
    hipLaunchKernelGGL((grouped_attn_tile_kernel<DS, FAR>), dim3(tiles, d.kv_heads), dim3(256), lds, s, d, b, v);
    FH_CHECK_LAUNCH();
    return 0;
}
template <int DS, bool FAR>
static int grouped_keys(const GroupedDims& d, const GroupedBuffers<bf16>& b, const BatchView& v, hipStream_t s) {
    constexpr size_t lds = (size_t)64 * (32 * DS + 4) * 4;
    static bool attr = false;
    if (!attr) { FH_CHECK_HIP(hipFuncSetAttribute((const void*)grouped_attn_keys_kernel<DS, FAR>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds)); attr = true; }
    const int G = d.heads / d.kv_heads, tiles = v.single ? v.num_seqs * cdiv(G, 16) : (int)((long)v.T * G / 16) + v.num_seqs;
    // split the keys while the launch has fewer workgroups than stay resident and a split keeps ≥ 128 keys
    const int keys = (int)std::min<long>(v.max_keys, (long)d.window + 16);
    int ns = 1;
    while (ns < 16 && tiles * d.kv_heads * ns < 512 && keys >= 2 * ns * 128) ns *= 2;
    if (knobs().grouped_splits > 0) ns = std::min(16, knobs().grouped_splits);
    while (ns > 1 && (size_t)tiles * d.kv_heads * ns * 16 * (d.vp + GROUPED_PARTIAL_PAD) * 4 > b.partial_bytes) ns /= 2;
    form_hit(ns > 1 ? FORM_GROUPED_ATTN_SPLIT : FORM_GROUPED_ATTN_KEYS);
    hipLaunchKernelGGL((grouped_attn_keys_kernel<DS, FAR>), dim3(tiles * ns, d.kv_heads), dim3(256), lds, s, d, b, v, ns);
    FH_CHECK_LAUNCH();
    if (ns > 1) {
        hipLaunchKernelGGL(grouped_attn_reduce_kernel, dim3(tiles, d.kv_heads), dim3(256), 0, s, d, b, v, ns);
        FH_CHECK_LAUNCH();
    }
    return 0;
}
template <> int grouped_attention<float>(const GroupedDims& d, const GroupedBuffers<float>& b, const BatchView& v, hipStream_t s) {
    return b.talk ? talking_attention(d, b, v, s) : grouped_plain(d, b, v, s);
}
template <> int grouped_attention<bf16>(const GroupedDims& d, const GroupedBuffers<bf16>& b, const BatchView& v, hipStream_t s) {
    if (b.talk) return talking_attention(d, b, v, s);
    if (knobs().grouped_plain || d.dp != d.vp || d.dp > 256 || d.scale <= 0.f) return grouped_plain(d, b, v, s);
    const bool tile = !v.single && (long)v.T * (d.heads / d.kv_heads) >= (long)knobs().grouped_tile_min_rows * v.num_seqs;
#define GROUPED(DS) \
    (b.r1 ? tile ? grouped_tile<DS, true>(d, b, v, s) : grouped_keys<DS, true>(d, b, v, s) : tile ? grouped_tile<DS, false>(d, b, v, s) : grouped_keys<DS, false>(d, b, v, s))
    switch (d.dp / 32) {
    case 1: return GROUPED(1);
    case 2: return GROUPED(2);
    case 3: return GROUPED(3);
    case 4: return GROUPED(4);
    case 6: return GROUPED(6);
    default: return GROUPED(8);
    }
#undef GROUPED
}
template int grouped_prepare<bf16>(const GroupedDims&, const GroupedBuffers<bf16>&, const BatchView&, hipStream_t);
template int grouped_prepare<float>(const GroupedDims&, const GroupedBuffers<float>&, const BatchView&, hipStream_t);

}  // namespace fh
