// Grouped attention whose heads' weights are mixed between softmax and values: weight_h(i, j) = Σ_g talk[h][g] · softmax_g(i, j), applied to
// the values of head h's own key / value head.  Caches, norms and queries are grouped_attention.hip's.
//
// The mixture needs every head's denominator before the first value is weighed.  Three forms:
//   plain  any size, both number formats: a workgroup per token, statistics first, then weights, mixture and values.
//   keys   few tokens: Σ_g talk[h][g] Σ_j softmax_g(j) v(j) — every head takes the values of EVERY key / value head with its own online
//          softmax in one pass over the cache, and the results are mixed at the end, in fp32, where the splits of the keys meet.
//   tile   portions: one pass over the keys for the statistics, a second one for weights, mixture (matrix cores, weights as the sum of two
//          16-bit numbers, so to 2⁻¹⁷) and values.
// Scores are in base 2 in the latter two.
#include <math.h>

#include <algorithm>

#include "common.h"
#include "grouped_cache.h"
#include "knobs.h"
#include "layer_ops.h"
#include "seq_tiles.h"

namespace fh {

namespace {

constexpr float LOG2E = 1.4426950408889634f;
constexpr int TALK_MAX_HEADS = 32;               // of the matrix-core forms
constexpr int TALK_TILE_SPLITS = 8;

// ── plain ──
template <typename E>
__global__ __launch_bounds__(256) void talk_attn_plain_kernel(GroupedDims d, GroupedBuffers<E> p, BatchView v) {
    typedef typename Frag<E>::v8 v8;
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int t = blockIdx.x, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, H = d.heads, G = H / d.kv_heads;
    float *q = lds, *wt = q + H * d.dp, *mixed = wt + H * 64, *o = mixed + H * 64;       // [H][dp], [H][64], [H][64], [H][vp]
    const int seq = v.tok_seq[t], pos = v.pos[seq] + t - v.cu[seq], lo = max(0, pos + 1 - d.window), hi = pos + 1;
    const int32_t* bt = v.bt + (long)seq * v.max_blocks;
    for (int i = tid; i < H * d.dp; i += 256) q[i] = (float)p.q[(long)t * H * d.dp + i];
    for (int i = tid; i < H * d.vp; i += 256) o[i] = 0.f;
    __syncthreads();
    auto score = [&](int h, int key) {
        if (key >= hi) return -INFINITY;
        const E* kt = p.k_pool + ((long)bt[key / 16] * d.kv_heads + h / G) * d.dp * 16 + (key % 16) * 8;
        float acc = 0.f;
        for (int i = 0; i < d.dp; i += 8) {
            const v8 x = *reinterpret_cast<const v8*>(kt + i * 16);
#pragma unroll
            for (int j = 0; j < 8; j++) acc += q[h * d.dp + i + j] * (float)x[j];
        }
        return acc * d.scale;
    };
    float *top = o + H * d.vp, *sum = top + H;                                           // [H] each
    for (int h = wave; h < H; h += 4) {
        float m = -INFINITY, l = 0.f;
        for (int k0 = lo; k0 < hi; k0 += 64) {
            const float sc = score(h, k0 + lane), m_new = fmaxf(m, wave_reduce_max(sc));
            l = l * expf(m - m_new) + wave_reduce_sum(expf(sc - m_new));
            m = m_new;
        }
        if (p.sink) l += expf(p.sink[h] - m);
        if (lane == 0) { top[h] = m; sum[h] = l; }
    }
    __syncthreads();
    for (int k0 = lo; k0 < hi; k0 += 64) {
        for (int h = wave; h < H; h += 4) wt[h * 64 + lane] = expf(score(h, k0 + lane) - top[h]) / sum[h];
        __syncthreads();
        for (int i = tid; i < H * 64; i += 256) {
            const int h = i >> 6;
            float acc = 0.f;
            for (int g = 0; g < H; g++) acc += p.talk[h * H + g] * wt[g * 64 + (i & 63)];
            mixed[i] = acc;
        }
        __syncthreads();
        const int n = min(64, hi - k0);
        for (int i = tid; i < H * d.vp; i += 256) {
            const int h = i / d.vp, c = i - h * d.vp;
            float acc = o[i];
            for (int k = 0; k < n; k++) {
                const int key = k0 + k;
                acc += mixed[h * 64 + k] * (float)p.v_pool[((long)bt[key / 16] * d.kv_heads + h / G) * d.vp * 16 + value_offset(key % 16, c)];
            }
            o[i] = acc;
        }
    }
    for (int i = tid; i < H * d.vp; i += 256) {                                          // (a thread's own elements)
        float f = p.mult;
        if (p.gate) f *= (float)p.gate[t * p.ld_gate + i / d.vp];
        if (p.value_gate) f *= (float)p.value_gate[t * p.ld_value_gate + i];
        p.out[(long)t * p.ldo + i] = (E)(o[i] * f);
    }
}

// ── keys ──
// grid (tokens × KV splits); wave w holds key / value heads w, w + NW, …: it scores their own query heads (columns of Sᵀ), hands the weights
// to everyone through LDS, and weighs its heads' values with the weights of all 16·HB query heads.  32 keys per step, one barrier; keys and
// values of the next step are on their way while this one is worked on.
// Partial of a (token, split): [16·HB heads][kv_heads·D] outputs, then maximum and sum per head.
template <int DS, int HB, int NW, int CW>
__global__ __launch_bounds__(64 * NW) void talk_attn_keys_kernel(GroupedDims d, GroupedBuffers<bf16> p, BatchView v, int t0, int nsplit) {
    constexpr int DT = 2 * DS, D = 32 * DS, HP = 16 * HB;
    __shared__ __attribute__((aligned(16))) bf16 lds_p[2][HP][4][8];
    __shared__ float lds_a[2][HP];
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63, a = lane >> 4, b = lane & 15;
    const int split = blockIdx.x % nsplit, unit = blockIdx.x / nsplit, tok = t0 + unit, G = d.heads / d.kv_heads;
    const int seq = __builtin_amdgcn_readfirstlane(v.single ? tok : v.tok_seq[tok]);
    const int row_pos = __builtin_amdgcn_readfirstlane((int)v.pos[seq] + tok - (int)v.cu[seq]), win_lo = max(0, row_pos + 1 - d.window);
    const int blk_lo = win_lo / 16, blk_hi = row_pos / 16 + 1, nstep = (blk_hi - blk_lo + 1) / 2;
    const int st_lo = nstep * split / nsplit, st_hi = nstep * (split + 1) / nsplit;
    const int32_t* bt = v.bt + (long)seq * v.max_blocks;
    const float sl2 = d.scale * LOG2E;
    const long kd = (long)d.kv_heads * D * 16;
    for (int i = threadIdx.x; i < 2 * HP * 32; i += 64 * NW) (&lds_p[0][0][0][0])[i] = (bf16)0.f;
    for (int i = threadIdx.x; i < 2 * HP; i += 64 * NW) (&lds_a[0][0])[i] = 1.f;
    bf16x8 qf[CW][DS], kf[CW][2][DS], vf[CW][2][DS];
    const bf16x8 zero = {};
    bool live[CW];
    long off[CW];
#pragma unroll
    for (int c = 0; c < CW; c++) {
        const int kvh = wave + NW * c;
        live[c] = kvh < d.kv_heads;
        off[c] = (long)min(kvh, d.kv_heads - 1) * D * 16 + lane * 8;
        const int head = min(kvh * G + min(b, G - 1), d.heads - 1);
#pragma unroll
        for (int s = 0; s < DS; s++) {
            const bf16x8 q = *reinterpret_cast<const bf16x8*>(p.q + ((long)tok * d.heads + head) * D + 32 * s + 8 * a);
            qf[c][s] = live[c] && b < G ? q : zero;
        }
    }
    // (past the end: a copy of the last block, masked)
    auto block_of = [&](int st, int i) { return (long)__builtin_amdgcn_readfirstlane(bt[min(blk_lo + 2 * st + i, blk_hi - 1)]); };
    auto load = [&](bf16x8 (&f)[CW][2][DS], const bf16* pool, const long (&blk)[2]) {
#pragma unroll
        for (int c = 0; c < CW; c++)
#pragma unroll
            for (int i = 0; i < 2; i++)
#pragma unroll
                for (int s = 0; s < DS; s++) f[c][i][s] = *reinterpret_cast<const bf16x8*>(pool + blk[i] * kd + off[c] + s * 512);
    };
    float m_run[CW], l_run[CW];
    floatx4 o[HB][CW][DT];
#pragma unroll
    for (int c = 0; c < CW; c++) {
        m_run[c] = -INFINITY; l_run[c] = 0.f;
#pragma unroll
        for (int h = 0; h < HB; h++)
#pragma unroll
            for (int t = 0; t < DT; t++) o[h][c][t] = (floatx4){0.f, 0.f, 0.f, 0.f};
    }
    long blk[2] = {block_of(st_lo, 0), block_of(st_lo, 1)};
    load(kf, p.k_pool, blk);
    load(vf, p.v_pool, blk);
    blk[0] = block_of(st_lo + 1, 0); blk[1] = block_of(st_lo + 1, 1);
    __syncthreads();
    for (int st = st_lo; st < st_hi; st++) {
        const int buf = st & 1;
#pragma unroll
        for (int c = 0; c < CW; c++) {
            float sc[8], mx = -INFINITY;
#pragma unroll
            for (int i = 0; i < 2; i++) {
                floatx4 s2[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
                for (int s = 0; s < DS; s++) s2[s & 1] = Frag<bf16>::mma(kf[c][i][s], qf[c][s], s2[s & 1]);
#pragma unroll
                for (int r = 0; r < 4; r++) {
                    const int key = (blk_lo + 2 * st + i) * 16 + 4 * a + r;
                    sc[4 * i + r] = key <= row_pos && key >= win_lo ? (s2[0][r] + s2[1][r]) * sl2 : -INFINITY;
                    mx = fmaxf(mx, sc[4 * i + r]);
                }
            }
            const float m_new = fmaxf(m_run[c], rows_reduce_max(mx)), m_safe = m_new == -INFINITY ? 0.f : m_new, alpha = __builtin_amdgcn_exp2f(m_run[c] - m_safe);
            bf16x8 pf;
            float ps = 0.f;
#pragma unroll
            for (int j = 0; j < 8; j++) { const float e = __builtin_amdgcn_exp2f(sc[j] - m_safe); ps += e; pf[j] = (bf16)e; }
            l_run[c] = l_run[c] * alpha + ps;                                  // (this lane's keys; the four lane groups meet at the end)
            m_run[c] = m_new;
            if (live[c] && b < G) {
                const int h = (wave + NW * c) * G + b;
                *reinterpret_cast<bf16x8*>(lds_p[buf][h][a]) = pf;
                if (a == 0) lds_a[buf][h] = alpha;
            }
        }
        load(kf, p.k_pool, blk);
        asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");        // (weights of step st; the other buffer's readers are past it)
#pragma unroll
        for (int h = 0; h < HB; h++) {
            const bf16x8 pf = *reinterpret_cast<const bf16x8*>(lds_p[buf][h * 16 + b][a]);
            const float alpha = lds_a[buf][h * 16 + b];
            const bool scaled = __ballot(alpha != 1.f) != 0;
#pragma unroll
            for (int c = 0; c < CW; c++)
#pragma unroll
                for (int t = 0; t < DT; t++) {
                    if (scaled)
#pragma unroll
                        for (int r = 0; r < 4; r++) o[h][c][t][r] *= alpha;
                    o[h][c][t] = Frag<bf16>::mma(value_operand(vf[c][0][t >> 1], vf[c][1][t >> 1], t & 1), pf, o[h][c][t]);
                }
        }
        load(vf, p.v_pool, blk);
        blk[0] = block_of(st + 2, 0); blk[1] = block_of(st + 2, 1);
    }
    const long kvd = (long)d.kv_heads * D;
    float* part = p.partial + (long)blockIdx.x * HP * (kvd + 2);
#pragma unroll
    for (int c = 0; c < CW; c++) {
        if (!live[c]) continue;
        const int kvh = wave + NW * c;
        const float l = rows_reduce_sum(l_run[c]);
        if (a == 0 && b < G) { part[HP * kvd + kvh * G + b] = m_run[c]; part[HP * (kvd + 1) + kvh * G + b] = l; }
#pragma unroll
        for (int h = 0; h < HB; h++)
#pragma unroll
            for (int t = 0; t < DT; t++)
                if (h * 16 + b < d.heads) *reinterpret_cast<floatx4*>(part + (h * 16 + b) * kvd + kvh * D + t * 16 + 4 * a) = o[h][c][t];
    }
}
// grid (tokens, kv_heads): the splits of every head's sum over this head's values, then the mixture
__global__ __launch_bounds__(256) void talk_attn_mix_kernel(GroupedDims d, GroupedBuffers<bf16> p, int t0, int nsplit, int hp) {
    extern __shared__ __attribute__((aligned(16))) float lds[];                // [heads][vp], factors [nsplit][heads], sums [nsplit][heads], rows of the mixture [G][heads]
    const int H = d.heads, G = H / d.kv_heads, kvh = blockIdx.y, D = d.vp, quads = D / 4;
    const long tok = t0 + blockIdx.x, kvd = (long)d.kv_heads * D, stride = hp * (kvd + 2);
    const float* part = p.partial + (long)blockIdx.x * nsplit * stride;
    float *f = lds + H * D, *sum = f + nsplit * H, *talk = sum + nsplit * H;
    for (int i = threadIdx.x; i < nsplit * H; i += 256) {
        const float* src = part + (i / H) * stride + hp * kvd + i % H;
        f[i] = src[0];
        sum[i] = src[hp];
    }
    for (int i = threadIdx.x; i < G * H; i += 256) talk[i] = p.talk[kvh * G * H + i] * p.mult;
    __syncthreads();
    for (int h = threadIdx.x; h < H; h += 256) {
        float M = -INFINITY, L = 0.f;
        for (int z = 0; z < nsplit; z++) M = fmaxf(M, f[z * H + h]);
        for (int z = 0; z < nsplit; z++) {
            const float e = __builtin_amdgcn_exp2f(f[z * H + h] - M);
            f[z * H + h] = e;
            L += sum[z * H + h] * e;
        }
        if (p.sink) L += __builtin_amdgcn_exp2f(p.sink[h] * LOG2E - M);
        const float inv = 1.0f / L;
        for (int z = 0; z < nsplit; z++) f[z * H + h] *= inv;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < H * quads; i += 256) {
        const int h = i / quads, c = (i - h * quads) * 4;
        const float* src = part + h * kvd + kvh * D + c;
        floatx4 x = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
        for (int z = 0; z < nsplit; z++) {
            const floatx4 y = *reinterpret_cast<const floatx4*>(src + z * stride);
            const float w = f[z * H + h];
#pragma unroll
            for (int r = 0; r < 4; r++) x[r] += y[r] * w;
        }
        *reinterpret_cast<floatx4*>(lds + h * D + c) = x;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < G * quads; i += 256) {
        const int g0 = i / quads, h = kvh * G + g0, c = (i - g0 * quads) * 4, col = h * D + c;
        float f1 = p.gate ? (float)p.gate[tok * p.ld_gate + h] : 1.f;
        bf16x4 y, gate = {(bf16)1.f, (bf16)1.f, (bf16)1.f, (bf16)1.f};
        if (p.value_gate) gate = *reinterpret_cast<const bf16x4*>(p.value_gate + tok * p.ld_value_gate + col);
        floatx4 x = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
        for (int g = 0; g < H; g++) {
            const floatx4 v = *reinterpret_cast<const floatx4*>(lds + g * D + c);
            const float w = talk[g0 * H + g];
#pragma unroll
            for (int r = 0; r < 4; r++) x[r] += w * v[r];
        }
#pragma unroll
        for (int r = 0; r < 4; r++) y[r] = (bf16)(x[r] * f1 * (float)gate[r]);
        *reinterpret_cast<bf16x4*>(p.out + tok * p.ldo + col) = y;
    }
}

// ── tile ──
// Statistics of the rows (token, query head of one key / value head): p.offset = maximum + log2(sum) with the sink, so that a weight is
// 2^(score − offset).  grid (128-row tiles, kv_heads): 4 waves × 2 tiles of 16 rows; 64 keys per step, wave w copies block w of the keys into LDS with
// the load unit, double-buffered.  A lane keeps the statistics of its own keys; the four lane groups meet at the end.
template <int DS>
__global__ __launch_bounds__(256) void talk_stats_kernel(GroupedDims d, GroupedBuffers<bf16> p, BatchView v, int min_tokens) {
    constexpr int MT = 2, D = 32 * DS, BLK = DS * 512;
    __shared__ __attribute__((aligned(16))) bf16 lds_k[2][4][BLK];
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63, a = lane >> 4, b = lane & 15;
    const int kvh = blockIdx.y, G = d.heads / d.kv_heads;
    SeqTile w;
    if (!find_seq_tile_last_first(v, G, 128, blockIdx.x, &w)) return;
    if (w.q_len < min_tokens) return;
    const int rows = w.q_len * G;
    const float sl2 = d.scale * LOG2E;
    bf16x8 qf[MT][DS];
    int row_pos[MT], win_lo[MT], vis_lo[MT], vis_hi[MT], head[MT];
    long tok[MT];
    bool ok[MT];
#pragma unroll
    for (int mt = 0; mt < MT; mt++) {
        const int r0 = w.tile * 128 + (wave * MT + mt) * 16, rho = min(r0 + b, rows - 1), tl = rho / G;
        ok[mt] = r0 + b < rows;
        head[mt] = kvh * G + rho - tl * G;
        tok[mt] = w.tok0 + tl;
        row_pos[mt] = w.pos0 + tl;
        win_lo[mt] = max(0, row_pos[mt] + 1 - d.window);
        vis_hi[mt] = w.pos0 + min(r0, rows - 1) / G;                           // keys in [vis_lo, vis_hi] are seen by every row of the tile
        vis_lo[mt] = max(0, w.pos0 + min(r0 + 15, rows - 1) / G + 1 - d.window);
#pragma unroll
        for (int s = 0; s < DS; s++) qf[mt][s] = *reinterpret_cast<const bf16x8*>(p.q + (tok[mt] * d.heads + head[mt]) * D + 8 * a + 32 * s);
    }
    const int t_first = w.tile * 128 / G, t_last = min(w.q_len - 1, (w.tile * 128 + 127) / G);
    const int blk_lo = max(0, w.pos0 + t_first + 1 - d.window) / 16, blk_hi = (w.pos0 + t_last + 16) / 16, nstep = (blk_hi - blk_lo + 3) / 4;
    const int32_t* bt = v.bt + (long)w.seq * v.max_blocks;
    const long kd = (long)d.kv_heads * D * 16, off = (long)kvh * D * 16 + lane * 8;
    auto block_of = [&](int st) { return (long)__builtin_amdgcn_readfirstlane(bt[min(blk_lo + 4 * st + wave, blk_hi - 1)]); };      // (past the end: a copy of the last, masked)
    auto issue = [&](long blk, int buf) {
#pragma unroll
        for (int s = 0; s < DS; s++)
            __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(p.k_pool + blk * kd + off + s * 512), (__attribute__((address_space(3))) void*)(lds_k[buf][wave] + s * 512), 16, 0, 0);
    };
    float m[MT], l[MT];
#pragma unroll
    for (int mt = 0; mt < MT; mt++) { m[mt] = -INFINITY; l[mt] = 0.f; }
    issue(block_of(0), 0);
    long next = block_of(1);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    for (int st = 0; st < nstep; st++) {
        const int buf = st & 1, key0 = (blk_lo + 4 * st) * 16;
        if (st + 1 < nstep) { issue(next, buf ^ 1); next = block_of(st + 2); }
        floatx4 sv[MT][4];
#pragma unroll
        for (int mt = 0; mt < MT; mt++)
#pragma unroll
            for (int i = 0; i < 4; i++) sv[mt][i] = (floatx4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < DS; s++)
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const bf16x8 k = *reinterpret_cast<const bf16x8*>(lds_k[buf][i] + s * 512 + lane * 8);
#pragma unroll
                for (int mt = 0; mt < MT; mt++) sv[mt][i] = Frag<bf16>::mma(k, qf[mt][s], sv[mt][i]);
            }
#pragma unroll
        for (int mt = 0; mt < MT; mt++) {
            if (!(key0 + 63 <= vis_hi[mt] && key0 >= vis_lo[mt])) {
#pragma unroll
                for (int i = 0; i < 4; i++)
#pragma unroll
                    for (int r = 0; r < 4; r++) {
                        const int key = key0 + i * 16 + 4 * a + r;
                        if (!(key <= row_pos[mt] && key >= win_lo[mt])) sv[mt][i][r] = -INFINITY;
                    }
            }
            float mx = -INFINITY;
#pragma unroll
            for (int i = 0; i < 4; i++) mx = fmaxf(mx, fmaxf(fmaxf(sv[mt][i][0], sv[mt][i][1]), fmaxf(sv[mt][i][2], sv[mt][i][3])));
            mx = fmaxf(m[mt], mx * sl2);                                       // (scale > 0, checked by the caller: the maximum commutes)
            const float safe = mx == -INFINITY ? 0.f : mx;
            float sum = l[mt] * __builtin_amdgcn_exp2f(m[mt] - safe);
#pragma unroll
            for (int i = 0; i < 4; i++)
#pragma unroll
                for (int r = 0; r < 4; r++) sum += __builtin_amdgcn_exp2f(__builtin_fmaf(sv[mt][i][r], sl2, -safe));
            m[mt] = mx;
            l[mt] = sum;
        }
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();
    }
#pragma unroll
    for (int mt = 0; mt < MT; mt++) {
        const float M = rows_reduce_max(m[mt]);                                // (a row sees itself: finite)
        float L = rows_reduce_sum(l[mt] * __builtin_amdgcn_exp2f(m[mt] - M));
        if (p.sink) L += __builtin_amdgcn_exp2f(p.sink[head[mt]] * LOG2E - M);
        if (ok[mt] && a == 0) p.offset[tok[mt] * d.heads + head[mt]] = M + __builtin_amdgcn_logf(L);
    }
}

// Weights, mixture and values.  grid (tiles of 16 tokens): eight waves of 2·HB heads each.  A step takes 32 keys: scores and weights of a wave's
// heads → LDS rows per (key, token), every weight as two 16-bit numbers; mixture of four keys per wave → LDS rows per (head, token);
// values of a wave's heads.  Rows are stored with their 16-byte chunks permuted by the token, so that neither side of the exchange meets in a bank.
// SHARED: the heads of a wave take their keys and values from one key / value head.
template <int DS, int HB, bool SHARED>
__global__ __launch_bounds__(512, 2) void talk_attn_tile_kernel(GroupedDims d, GroupedBuffers<bf16> p, BatchView v, int min_tokens, int nsplit) {
    constexpr int DT = 2 * DS, D = 32 * DS, HP = 16 * HB, HPW = 2 * HB, KS = HB, CH = 4 * HB;      // CH: 16-byte chunks of a (key, token) row
    constexpr bool AHEAD = SHARED && HPW * DS <= 8;                            // registers for a step's values and the next one's keys on their way
    extern __shared__ __attribute__((aligned(16))) bf16 lds_x[];
    // [32 keys][16 tokens][CH][8], [HP][16 tokens][4][8], the mixing matrix as operands [HB][KS][64 lanes][8]
    bf16 *lw = lds_x, *lp = lw + 32 * 16 * CH * 8, *lt = lp + HP * 16 * 32;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63, a = lane >> 4, b = lane & 15;
    const int H = d.heads, G = H / d.kv_heads, h0 = wave * HPW;                // h0: this wave's first head
    SeqTile w;
    const int split = blockIdx.x % nsplit;
    if (!find_seq_tile_last_first(v, 1, 16, blockIdx.x / nsplit, &w)) return;
    if (w.q_len < min_tokens) return;
    const float sl2 = d.scale * LOG2E;
    const int32_t* bt = v.bt + (long)w.seq * v.max_blocks;
    const int t_first = w.tile * 16, t_last = min(w.q_len, t_first + 16) - 1, tl = min(t_first + b, t_last);
    const int blk_lo = max(0, w.pos0 + t_first + 1 - d.window) / 16, blk_hi = (w.pos0 + t_last) / 16 + 1, nstep = (blk_hi - blk_lo + 1) / 2;
    const int row_pos = w.pos0 + tl, win_lo = max(0, row_pos + 1 - d.window);
    const int all_lo = max(0, w.pos0 + t_last + 1 - d.window), all_hi = w.pos0 + t_first;       // keys that every row sees
    const long tok = w.tok0 + tl;
    bf16x8 qf[HPW][DS];
    float offset[HPW];
    int off[HPW];                                                              // of the head's keys (and values) in a block
#pragma unroll
    for (int i = 0; i < HPW; i++) {
        const int h = min(h0 + i, H - 1);                                      // (heads past the last one weigh nothing: their columns of the mixture are zero)
        offset[i] = p.offset[tok * H + h];
        off[i] = h / G * D * 16;
#pragma unroll
        for (int s = 0; s < DS; s++) qf[i][s] = *reinterpret_cast<const bf16x8*>(p.q + (tok * H + h) * D + 8 * a + 32 * s);
    }
    const long kd = (long)d.kv_heads * D * 16;
    const unsigned at = lane * 8;                                              // (scalar addresses plus this)
    auto block_of = [&](int st, int i) { return (long)__builtin_amdgcn_readfirstlane(bt[min(blk_lo + 2 * st + i, blk_hi - 1)]); };      // (past the end: a copy of the last, masked)
    // a (key, token) row holds, wave by wave, its heads' first halves and then their second halves
    for (int i = threadIdx.x; i < HB * KS * 512; i += 512) {
        const int m = i / (KS * 512), ks = i / 512 % KS, ln = i / 8 % 64, j = i % 8;
        const int h = m * 16 + (ln & 15), c = 4 * ks + (ln >> 4), g = HPW == 2 ? 4 * c + 2 * (j >> 2) + (j & 1) : 4 * c + (j & 3);
        lt[i] = (bf16)(h < H && g < H ? p.talk[h * H + g] : 0.f);
    }
    floatx4 o[HPW][DT];
#pragma unroll
    for (int i = 0; i < HPW; i++)
#pragma unroll
        for (int t = 0; t < DT; t++) o[i][t] = (floatx4){0.f, 0.f, 0.f, 0.f};
    const int wchunk = HPW == 2 ? wave >> 1 : wave, whalf = HPW == 2 ? (wave & 1) * 4 : 0;      // this wave's place in the (key, token) rows
    auto row_chunk = [&](int c) { return HB == 1 ? c ^ ((b >> 2) & 3) : c ^ (b & 7); };
    // a block's operands of the wave's first head (all its heads, where they share them)
    auto load = [&](bf16x8 (&f)[DS], const bf16* pool, long blk) {
#pragma unroll
        for (int s = 0; s < DS; s++) f[s] = *reinterpret_cast<const bf16x8*>(pool + (blk * kd + off[0] + s * 512) + at);
    };
    // weights of this wave's heads and one block of keys; kq: the keys, where they are there already
    auto weigh = [&](int k, int key0, long blk, const bf16x8 (&kq)[DS]) {
        floatx4 sc[HPW];
#pragma unroll
        for (int i = 0; i < HPW; i++) sc[i] = (floatx4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i0 = 0; i0 < HPW; i0 += SHARED ? HPW : 1)
#pragma unroll
            for (int s = 0; s < DS; s++) {
                const bf16x8 kf = AHEAD ? kq[s] : *reinterpret_cast<const bf16x8*>(p.k_pool + (blk * kd + off[i0] + s * 512) + at);
#pragma unroll
                for (int i = i0; i < (SHARED ? HPW : i0 + 1); i++) sc[i] = Frag<bf16>::mma(kf, qf[i][s], sc[i]);
            }
#pragma unroll
        for (int i = 0; i < HPW; i++)
#pragma unroll
            for (int r = 0; r < 4; r++) sc[i][r] = __builtin_amdgcn_exp2f(__builtin_fmaf(sc[i][r], sl2, -offset[i]));
        if (!(key0 >= all_lo && key0 + 15 <= all_hi)) {
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const int key = key0 + 4 * a + r;
                const bool seen = key <= row_pos && key >= win_lo;
#pragma unroll
                for (int i = 0; i < HPW; i++) sc[i][r] = seen ? sc[i][r] : 0.f;
            }
        }
#pragma unroll
        for (int r = 0; r < 4; r++) {
            typedef bf16 entries __attribute__((ext_vector_type(2 * HPW)));
            entries y;
#pragma unroll
            for (int i = 0; i < HPW; i++) {
                y[i] = (bf16)sc[i][r];
                y[HPW + i] = (bf16)(sc[i][r] - (float)y[i]);
            }
            *reinterpret_cast<entries*>(lw + ((k * 16 + 4 * a + r) * 16 + b) * CH * 8 + row_chunk(wchunk) * 8 + whalf) = y;
        }
    };
    // the mixture of four keys (`quad` of eight in the step).  A row ahead, 16 mixed heads at a time, products to 16 bits as soon as they are
    // there: registers are what this kernel is short of.
    auto mix = [&](int quad) {
        const bf16* row = lw + (quad * 4 * 16 + b) * CH * 8;
#pragma unroll
        for (int m = 0; m < HB; m++) {
            bf16x8 tf[KS], wf[2][KS];
            bf16x4 y[4];
#pragma unroll
            for (int ks = 0; ks < KS; ks++) {
                tf[ks] = *reinterpret_cast<const bf16x8*>(lt + ((m * KS + ks) * 64 + lane) * 8);
                wf[0][ks] = *reinterpret_cast<const bf16x8*>(row + row_chunk(4 * ks + a) * 8);
            }
#pragma unroll
            for (int r = 0; r < 4; r++) {
                if (r < 3)
#pragma unroll
                    for (int ks = 0; ks < KS; ks++) wf[(r + 1) & 1][ks] = *reinterpret_cast<const bf16x8*>(row + (r + 1) * 16 * CH * 8 + row_chunk(4 * ks + a) * 8);
                __builtin_amdgcn_sched_barrier(0);
                floatx4 x = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int ks = 0; ks < KS; ks++) x = Frag<bf16>::mma(tf[ks], wf[r & 1][ks], x);
#pragma unroll
                for (int q = 0; q < 4; q++) y[q][r] = (bf16)x[q];
            }
            // lane (a, b): heads 16·m + 4·a + q of token b, the four keys side by side
#pragma unroll
            for (int q = 0; q < 4; q++) *reinterpret_cast<bf16x4*>(lp + ((m * 16 + 4 * a + q) * 16 + b) * 32 + ((quad & 3) ^ ((b >> 2) & 3)) * 8 + (quad >> 2) * 4) = y[q];
        }
    };
    const int st_lo = nstep * split / nsplit, st_hi = nstep * (split + 1) / nsplit;
    long next0 = block_of(st_lo, 0), next1 = block_of(st_lo, 1);
    bf16x8 kq[2][DS], vq[2][DS];
    if (AHEAD) { load(kq[0], p.k_pool, next0); load(kq[1], p.k_pool, next1); }
    for (int st = st_lo; st < st_hi; st++) {
        const long blk0 = next0, blk1 = next1;
        const bf16 *v0 = p.v_pool + blk0 * kd, *v1 = p.v_pool + blk1 * kd;
        next0 = block_of(st + 1, 0);
        next1 = block_of(st + 1, 1);
        if (AHEAD) {
            load(vq[0], p.v_pool, blk0); load(vq[1], p.v_pool, blk1);
            __builtin_amdgcn_sched_barrier(0);
            weigh(0, (blk_lo + 2 * st) * 16, blk0, kq[0]);
            weigh(1, (blk_lo + 2 * st + 1) * 16, blk1, kq[1]);
            load(kq[0], p.k_pool, next0); load(kq[1], p.k_pool, next1);
        } else {
#pragma unroll 1
            for (int k = 0; k < 2; k++) weigh(k, (blk_lo + 2 * st + k) * 16, k ? blk1 : blk0, kq[0]);
        }
        asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
        mix(wave);
        asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
        bf16x8 pf[HPW];
#pragma unroll
        for (int i = 0; i < HPW; i++) pf[i] = *reinterpret_cast<const bf16x8*>(lp + ((h0 + i) * 16 + b) * 32 + (a ^ ((b >> 2) & 3)) * 8);
        if (AHEAD) {
#pragma unroll
            for (int s = 0; s < DS; s++)
#pragma unroll
                for (int i = 0; i < HPW; i++)
#pragma unroll
                    for (int sub = 0; sub < 2; sub++) o[i][2 * s + sub] = Frag<bf16>::mma(value_operand(vq[0][s], vq[1][s], sub), pf[i], o[i][2 * s + sub]);
        } else if (SHARED) {
            bf16x8 vf[2][2];
            vf[0][0] = *reinterpret_cast<const bf16x8*>(v0 + off[0] + at);
            vf[0][1] = *reinterpret_cast<const bf16x8*>(v1 + off[0] + at);
#pragma unroll
            for (int s = 0; s < DS; s++) {
                if (s + 1 < DS) {
                    vf[(s + 1) & 1][0] = *reinterpret_cast<const bf16x8*>(v0 + off[0] + (s + 1) * 512 + at);
                    vf[(s + 1) & 1][1] = *reinterpret_cast<const bf16x8*>(v1 + off[0] + (s + 1) * 512 + at);
                }
                __builtin_amdgcn_sched_barrier(0);
#pragma unroll
                for (int i = 0; i < HPW; i++)
#pragma unroll
                    for (int sub = 0; sub < 2; sub++) o[i][2 * s + sub] = Frag<bf16>::mma(value_operand(vf[s & 1][0], vf[s & 1][1], sub), pf[i], o[i][2 * s + sub]);
            }
        } else {
#pragma unroll
            for (int i = 0; i < HPW; i++)
#pragma unroll
                for (int s = 0; s < DS; s++) {
                    const bf16x8 x0 = *reinterpret_cast<const bf16x8*>(v0 + off[i] + s * 512 + at), x1 = *reinterpret_cast<const bf16x8*>(v1 + off[i] + s * 512 + at);
                    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
                    for (int sub = 0; sub < 2; sub++) o[i][2 * s + sub] = Frag<bf16>::mma(value_operand(x0, x1, sub), pf[i], o[i][2 * s + sub]);
                }
        }
    }
    if (t_first + b > t_last) return;
    if (nsplit > 1) {                                                          // [splits][T][heads·D], to be summed
        float* part = p.partial + ((long)split * v.T + tok) * H * D;
#pragma unroll
        for (int i = 0; i < HPW; i++) {
            if (h0 + i >= H) break;
#pragma unroll
            for (int t = 0; t < DT; t++) *reinterpret_cast<floatx4*>(part + (h0 + i) * D + t * 16 + 4 * a) = o[i][t];
        }
        return;
    }
#pragma unroll
    for (int i = 0; i < HPW; i++) {
        if (h0 + i >= H) break;
        float f = p.mult;
        if (p.gate) f *= (float)p.gate[tok * p.ld_gate + h0 + i];
#pragma unroll
        for (int t = 0; t < DT; t++) {
            const int col = (h0 + i) * D + t * 16 + 4 * a;
            bf16x4 y, g = {(bf16)1.f, (bf16)1.f, (bf16)1.f, (bf16)1.f};
            if (p.value_gate) g = *reinterpret_cast<const bf16x4*>(p.value_gate + tok * p.ld_value_gate + col);
#pragma unroll
            for (int r = 0; r < 4; r++) y[r] = (bf16)(o[i][t][r] * f * (float)g[r]);
            *reinterpret_cast<bf16x4*>(p.out + tok * p.ldo + col) = y;
        }
    }
}

// the key splits of a token of a portion, times the gates
__global__ __launch_bounds__(256) void talk_attn_sum_kernel(GroupedDims d, GroupedBuffers<bf16> p, BatchView v, int min_tokens, int nsplit) {
    const int t = blockIdx.x, seq = v.tok_seq[t], cols = d.heads * d.vp;
    if ((int)(v.cu[seq + 1] - v.cu[seq]) < min_tokens) return;
    for (int c = threadIdx.x * 4; c < cols; c += 1024) {
        const float* src = p.partial + (long)t * cols + c;
        floatx4 x = *reinterpret_cast<const floatx4*>(src);
        for (int z = 1; z < nsplit; z++) x += *reinterpret_cast<const floatx4*>(src + (long)z * v.T * cols);
        float f = p.mult;
        if (p.gate) f *= (float)p.gate[t * p.ld_gate + c / d.vp];
        bf16x4 y, g = {(bf16)1.f, (bf16)1.f, (bf16)1.f, (bf16)1.f};
        if (p.value_gate) g = *reinterpret_cast<const bf16x4*>(p.value_gate + t * p.ld_value_gate + c);
#pragma unroll
        for (int r = 0; r < 4; r++) y[r] = (bf16)(x[r] * f * (float)g[r]);
        *reinterpret_cast<bf16x4*>(p.out + (long)t * p.ldo + c) = y;
    }
}

template <typename E>
int talk_plain(const GroupedDims& d, const GroupedBuffers<E>& b, const BatchView& v, hipStream_t s) {
    form_hit(FORM_TALK_ATTN_PLAIN);
    const size_t lds = (size_t)d.heads * (d.dp + d.vp + 128 + 2) * 4;
    FH_REQUIRE(lds <= 160 * 1024, "attention with mixed heads: %d heads of %d / %d do not fit LDS", d.heads, d.dim, d.vdim);
    static bool attr = false;
    if (!attr) { FH_CHECK_HIP(hipFuncSetAttribute((const void*)talk_attn_plain_kernel<E>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024)); attr = true; }
    hipLaunchKernelGGL(talk_attn_plain_kernel<E>, dim3(v.T), dim3(256), lds, s, d, b, v);
    FH_CHECK_LAUNCH();
    return 0;
}

size_t talk_partial(const GroupedDims& d) { return (size_t)(d.heads <= 16 ? 16 : 32) * ((size_t)d.kv_heads * d.vp + 2) * 4; }
bool talk_tile_supports(const GroupedDims& d) {
    return d.heads <= TALK_MAX_HEADS && d.dp == d.vp && d.dp <= (d.heads <= 16 ? 256 : 128) && d.scale > 0.f;
}
// (registers: query heads of two row tiles, or two key / value heads per wave, up to 128 dimensions)
bool talk_keys_supports(const GroupedDims& d) {
    return talk_tile_supports(d) && d.heads / d.kv_heads <= 16 && d.kv_heads <= (d.heads <= 16 && d.dp <= 128 ? 16 : 8);
}
template <int DS, int HB, bool SHARED>
int talk_tile(const GroupedDims& d, const GroupedBuffers<bf16>& b, const BatchView& v, int min_tokens, hipStream_t s) {
    constexpr size_t lds = ((size_t)32 * 16 * 4 * HB * 8 + (size_t)16 * HB * 16 * 32 + HB * HB * 512) * 2;
    static bool attr = false;
    if (!attr) { FH_CHECK_HIP(hipFuncSetAttribute((const void*)talk_attn_tile_kernel<DS, HB, SHARED>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds)); attr = true; }
    const int tiles = v.single ? v.num_seqs : v.T / 16 + v.num_seqs;              // upper bound of Σ ceil(tokens of a sequence / rows)
    form_hit(FORM_TALK_ATTN_TILE);
    const int G = d.heads / d.kv_heads, stats = v.single ? v.num_seqs * cdiv(G, 128) : (int)((long)v.T * G / 128) + v.num_seqs;
    hipLaunchKernelGGL((talk_stats_kernel<DS>), dim3(stats, d.kv_heads), dim3(256), 0, s, d, b, v, min_tokens);
    FH_CHECK_LAUNCH();
    // split the keys while the launch has fewer workgroups than two per CU and a split of the longest context keeps ≥ 8 steps: the tiles of one
    // long portion differ in length, and few of them leave CUs without work
    const int keys = (int)std::min<long>(v.max_keys, (long)d.window + 16);
    const size_t row_bytes = (size_t)v.T * d.heads * d.vp * 4;
    int ns = 1;
    while (ns < TALK_TILE_SPLITS && tiles * ns < 512 && keys >= 2 * ns * 256) ns *= 2;
    if (knobs().talk_tile_splits > 0) ns = std::min(TALK_TILE_SPLITS, knobs().talk_tile_splits);
    while (ns > 1 && ns * row_bytes > b.partial_bytes) ns /= 2;
    hipLaunchKernelGGL((talk_attn_tile_kernel<DS, HB, SHARED>), dim3(tiles * ns), dim3(512), lds, s, d, b, v, min_tokens, ns);
    FH_CHECK_LAUNCH();
    if (ns > 1) {
        form_hit(FORM_TALK_ATTN_TILE_SPLIT);
        hipLaunchKernelGGL(talk_attn_sum_kernel, dim3(v.T), dim3(256), 0, s, d, b, v, min_tokens, ns);
        FH_CHECK_LAUNCH();
    }
    return 0;
}
// tokens [t0, t0 + n) of the batch
template <int DS, int HB>
int talk_keys(const GroupedDims& d, const GroupedBuffers<bf16>& b, const BatchView& v, int t0, int n, hipStream_t s) {
    const int keys = (int)std::min<long>(v.max_keys, (long)d.window + 16), room = (int)(b.partial_bytes / talk_partial(d)), hp = 16 * HB;
    FH_REQUIRE(room > 0, "attention with mixed heads: no scratch");
    form_hit(FORM_TALK_ATTN_KEYS);
    for (int done = 0; done < n;) {
        const int m = std::min(n - done, room);
        // split the keys while the launch has fewer workgroups than stay resident and a split keeps ≥ 128 keys
        int ns = 1;
        while (ns < 64 && m * ns < 512 && keys >= 2 * ns * 128) ns *= 2;
        if (knobs().grouped_splits > 0) ns = std::min(64, knobs().grouped_splits);
        while (ns > 1 && m * ns > room) ns /= 2;
        const dim3 grid(m * ns);
#define KEYS(NW, CW) hipLaunchKernelGGL((talk_attn_keys_kernel<DS, HB, NW, CW>), grid, dim3(64 * NW), 0, s, d, b, v, t0 + done, ns)
        if (d.kv_heads <= 4) KEYS(4, 1);
        else if (d.kv_heads <= 8) KEYS(8, 1);
        else if constexpr (HB == 1 && DS <= 4) KEYS(8, 2);
#undef KEYS
        FH_CHECK_LAUNCH();
        hipLaunchKernelGGL(talk_attn_mix_kernel, dim3(m, d.kv_heads), dim3(256), (size_t)d.heads * (d.vp + 2 * ns + d.heads / d.kv_heads) * 4, s, d, b, t0 + done, ns, hp);
        FH_CHECK_LAUNCH();
        done += m;
    }
    return 0;
}
template <int DS, int HB>
int talk_tile(const GroupedDims& d, const GroupedBuffers<bf16>& b, const BatchView& v, int min_tokens, hipStream_t s) {
    return d.heads / d.kv_heads % (2 * HB) == 0 ? talk_tile<DS, HB, true>(d, b, v, min_tokens, s) : talk_tile<DS, HB, false>(d, b, v, min_tokens, s);
}
template <int DS, int HB>
int talk_forms(const GroupedDims& d, const GroupedBuffers<bf16>& b, const BatchView& v, hipStream_t s) {
    const int min_tokens = knobs().talk_tile_min_tokens;
    if (!talk_keys_supports(d)) return talk_tile<DS, HB>(d, b, v, 0, s);
    if (v.single || min_tokens <= 0) return talk_keys<DS, HB>(d, b, v, 0, v.T, s);
    // runs of sequences with few tokens, then everything else in one launch
    bool any_long = false;
    for (int i = 0; i < v.num_seqs;) {
        int j = i;
        while (j < v.num_seqs && (int)(v.host_cu[j + 1] - v.host_cu[j]) < min_tokens) j++;
        if (j > i)
            if (int rc = talk_keys<DS, HB>(d, b, v, (int)v.host_cu[i], (int)(v.host_cu[j] - v.host_cu[i]), s)) return rc;
        if (j < v.num_seqs) { any_long = true; j++; }
        i = j;
    }
    return any_long ? talk_tile<DS, HB>(d, b, v, min_tokens, s) : 0;
}

}  // namespace

size_t talking_partial_bytes(const GroupedDims& d, int max_tokens) {
    // 512 (token, split) pairs of the keys form; key splits of the tile form, which has fewer than 512 tiles where it splits
    const size_t keys = talk_keys_supports(d) ? 512 * talk_partial(d) : 0;
    const size_t rows = std::min<size_t>((size_t)TALK_TILE_SPLITS * max_tokens, 1024 * 16);
    return std::max(keys, talk_tile_supports(d) ? rows * d.heads * d.vp * 4 : 0);
}

template <> int talking_attention<float>(const GroupedDims& d, const GroupedBuffers<float>& b, const BatchView& v, hipStream_t s) { return talk_plain(d, b, v, s); }
template <> int talking_attention<bf16>(const GroupedDims& d, const GroupedBuffers<bf16>& b, const BatchView& v, hipStream_t s) {
    if (knobs().grouped_plain || !talk_tile_supports(d)) return talk_plain(d, b, v, s);
    if (d.heads > 16) {
        switch (d.dp / 32) {
        case 1: return talk_forms<1, 2>(d, b, v, s);
        case 2: return talk_forms<2, 2>(d, b, v, s);
        case 3: return talk_forms<3, 2>(d, b, v, s);
        default: return talk_forms<4, 2>(d, b, v, s);
        }
    }
    switch (d.dp / 32) {
    case 1: return talk_forms<1, 1>(d, b, v, s);
    case 2: return talk_forms<2, 1>(d, b, v, s);
    case 3: return talk_forms<3, 1>(d, b, v, s);
    case 4: return talk_forms<4, 1>(d, b, v, s);
    case 6: return talk_forms<6, 1>(d, b, v, s);
    default: return talk_forms<8, 1>(d, b, v, s);
    }
}

}  // namespace fh
