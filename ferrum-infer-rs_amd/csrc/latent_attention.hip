// Attention over a compressed cache (multi-head latent attention): a token caches one normed latent c and one rotated key part shared
// by all heads; head h's key is (W_uk,h c | shared part) and its value W_uv,h c.
//
// The kernels here never expand keys or values: the query's plain part arrives already multiplied by W_uk,hᵀ (q_lat), so a score is
// q_lat · c + rot(q) · k_rot, and the output is left in latent space (o_lat = Σ p c) for the value projection that follows.  All heads
// of a token share one cache entry, so a 16-row MFMA tile is 16 (token, head) pairs of one sequence and the cache is read once for them.
//
// Cache tiles are K-fragment shaped ([chunk of 8 dims][16 keys][8]): a wave's K fragment is one contiguous 1-KiB load and feeds the
// matrix pipe directly.  The same registers are parked in wave-private LDS and come back transposed (ds_read_b64_tr_b16) as the Vᵀ
// operand of O ᵀ += Vᵀ·Pᵀ — the latent is read from memory once for both products.
#include <math.h>

#include <algorithm>

#include "common.h"
#include "knobs.h"
#include "layer_ops.h"

namespace fh {

// rotate the pairs (2i, 2i + 1) of 8 consecutive values starting at dimension d0, position `pos`; dims past rot_dims pass
template <typename V>
__device__ __forceinline__ V rotate8(V x, int d0, int rot_dims, const float* __restrict__ cos_t, const float* __restrict__ sin_t, long pos) {
    const int half = rot_dims >> 1;
#pragma unroll
    for (int j = 0; j < 4; j++) {
        const int i = (d0 >> 1) + j;
        if (i < half) {
            const float c = cos_t[pos * half + i], s = sin_t[pos * half + i], u = (float)x[2 * j], w = (float)x[2 * j + 1];
            x[2 * j] = u * c - w * s;
            x[2 * j + 1] = w * c + u * s;
        }
    }
    return x;
}

// one wave per token: norm of the query latent, norm of the kv latent, rotation of the shared key part, cache write
template <typename E>
__global__ __launch_bounds__(256) void latent_prepare_kernel(const E* __restrict__ dq, const E* __restrict__ dkv, long ld,
                                                             const float* __restrict__ dq_norm, const float* __restrict__ dkv_norm,
                                                             float eps, LatentDims d, LatentBuffers<E> b, BatchView v, E* __restrict__ cq) {
    typedef typename Frag<E>::v8 v8;
    const int t = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (t >= v.T) return;
    const int seq = v.tok_seq[t];
    const long pos = (long)v.pos[seq] + t - v.cu[seq];
    const E *qr = dq + t * ld, *kr = dkv + t * ld;
    float sq = 0.f, sk = 0.f;
    for (int i = lane * 8; i < d.qp; i += 512) {
        const v8 x = *reinterpret_cast<const v8*>(qr + i);
#pragma unroll
        for (int j = 0; j < 8; j++) sq += (float)x[j] * (float)x[j];      // (padded columns are zero)
    }
    for (int i = lane * 8; i < d.kp; i += 512) {
        const v8 x = *reinterpret_cast<const v8*>(kr + i);
#pragma unroll
        for (int j = 0; j < 8; j++) sk += (float)x[j] * (float)x[j];
    }
    const float iq = 1.0f / sqrtf(wave_reduce_sum(sq) / (float)d.q_rank + eps), ik = 1.0f / sqrtf(wave_reduce_sum(sk) / (float)d.kv_rank + eps);
    for (int i = lane * 8; i < d.qp; i += 512) {
        v8 x = *reinterpret_cast<const v8*>(qr + i);
#pragma unroll
        for (int j = 0; j < 8; j++) x[j] = (E)((float)x[j] * iq * dq_norm[i + j]);
        *reinterpret_cast<v8*>(cq + (long)t * d.qp + i) = x;
    }
    E* tile = b.pool + (long)v.bt[(long)seq * v.max_blocks + pos / 16] * 16 * (d.kp + d.rp) + (pos % 16) * 8;
    for (int i = lane * 8; i < d.kp + d.rp; i += 512) {
        v8 x = *reinterpret_cast<const v8*>(kr + i);
        if (i < d.kp) {
#pragma unroll
            for (int j = 0; j < 8; j++) x[j] = (E)((float)x[j] * ik * dkv_norm[i + j]);
        } else {
            x = rotate8(x, i - d.kp, d.rot_dims, b.cos_t, b.sin_t, pos);
        }
        *reinterpret_cast<v8*>(tile + i * 16) = x;
    }
}

template <typename E>
int latent_prepare(const E* dq, const E* dkv, long ld, const float* dq_norm, const float* dkv_norm, float eps, const LatentDims& d,
                   const LatentBuffers<E>& b, const BatchView& v, E* cq, hipStream_t s) {
    hipLaunchKernelGGL(latent_prepare_kernel<E>, dim3(cdiv(v.T, 4)), dim3(256), 0, s, dq, dkv, ld, dq_norm, dkv_norm, eps, d, b, v, cq);
    FH_CHECK_LAUNCH();
    return 0;
}

// ── plain form: one workgroup per (token, head), 256 keys at a time; any size, both number formats ──
template <typename E>
__global__ __launch_bounds__(256) void latent_attn_plain_kernel(LatentDims d, LatentBuffers<E> b, BatchView v) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, wave = tid >> 6, kd = d.kp + d.rp;
    float *q = lds, *pr = lds + kd, *red = pr + 256, *o = red + 8;         // [kd] query, [256] weights, [8], [kp] output
    const int seq = v.tok_seq[t];
    const int pos = v.pos[seq] + t - v.cu[seq];
    for (int i = tid; i < d.kp; i += 256) { q[i] = (float)b.q_lat[((long)t * d.heads + h) * d.kp + i]; o[i] = 0.f; }
    const E* qr = b.q + ((long)t * d.heads + h) * (d.dp + d.rp) + d.dp;
    const int half = d.rot_dims >> 1;
    for (int i = tid; i < d.rp; i += 256) {
        float x = (float)qr[i];
        if (i < d.rot_dims) {
            const float c = b.cos_t[(long)pos * half + i / 2], s = b.sin_t[(long)pos * half + i / 2], y = (float)qr[i ^ 1];
            x = i & 1 ? x * c + y * s : x * c - y * s;
        }
        q[d.kp + i] = x;
    }
    const int lo = max(0, pos + 1 - d.window), hi = pos + 1;
    const int32_t* bt = v.bt + (long)seq * v.max_blocks;
    float m_run = -INFINITY, l_run = 0.f;
    __syncthreads();
    for (int k0 = lo; k0 < hi; k0 += 256) {
        const int key = k0 + tid;
        float sc = -INFINITY;
        if (key < hi) {
            const E* kt = b.pool + (long)bt[key / 16] * 16 * kd + (key % 16) * 8;
            float acc = 0.f;
            for (int i = 0; i < kd; i += 8) {
                const typename Frag<E>::v8 x = *reinterpret_cast<const typename Frag<E>::v8*>(kt + i * 16);
#pragma unroll
                for (int j = 0; j < 8; j++) acc += q[i + j] * (float)x[j];
            }
            sc = acc * d.scale;
        }
        float mx = wave_reduce_max(sc);
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
        for (int i = tid; i < d.kp; i += 256) {
            float acc = o[i] * alpha;
            for (int k = 0; k < n; k++) {
                const int kk = k0 + k;
                acc += pr[k] * (float)b.pool[(long)bt[kk / 16] * 16 * kd + ((i >> 3) * 16 + kk % 16) * 8 + (i & 7)];
            }
            o[i] = acc;
        }
        __syncthreads();
    }
    for (int i = tid; i < d.kp; i += 256) b.o_lat[((long)t * d.heads + h) * d.kp + i] = (E)(o[i] / l_run);
}

// ── matrix-core form ──
struct LatentTile { int seq, tile, tok0, q_len, pos0; };
// 16-row tiles of (token, head) pairs, numbered sequence by sequence; every wave finds tile w by a scan of cu_seqlens
__device__ __forceinline__ bool find_latent_tile(const BatchView& v, int heads, int w, LatentTile* o) {
    const int lane = threadIdx.x & 63;
    int base = 0;
    for (int s0 = 0; s0 < v.num_seqs; s0 += 64) {
        const int s = s0 + lane;
        const int units = s < v.num_seqs ? ((int)(v.cu[s + 1] - v.cu[s]) * heads + 15) >> 4 : 0;
        int incl = units;
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
            const int t = __shfl_up(incl, off, 64);
            if (lane >= off) incl += t;
        }
        const int total = __shfl(incl, 63, 64);
        if (w < base + total) {
            const int src = __ffsll((unsigned long long)__ballot(w < base + incl)) - 1;
            o->seq = __builtin_amdgcn_readfirstlane(s0 + src);
            o->tile = __builtin_amdgcn_readfirstlane(w - (base + __shfl(incl - units, src, 64)));
            o->tok0 = (int)v.cu[o->seq];
            o->q_len = (int)v.cu[o->seq + 1] - o->tok0;
            o->pos0 = (int)v.pos[o->seq];
            return true;
        }
        base += total;
    }
    return false;
}

constexpr int LATENT_RS = 2;           // k-steps of the rotated part: rot_dim ≤ 64
constexpr int LATENT_PARTIAL_PAD = 4;  // floats behind a partial row's outputs: maximum, sum

// KS: most k-steps of the latent (kv_rank ≤ 32·KS).  grid (row tiles, KV splits), 4 waves over the keys of a split.
template <int KS>
__global__ __launch_bounds__(256, 1) void latent_attn_kernel(LatentDims d, LatentBuffers<bf16> p, BatchView v, int nsplit) {
    constexpr int DT = 2 * KS, OSTR = 32 * KS + 4;
    constexpr int STAGE = KS * 512;                                            // one 16-key block of latents per wave
    constexpr int LDS_BYTES = 4 * STAGE * 2 > 16 * OSTR * 4 ? 4 * STAGE * 2 : 16 * OSTR * 4;
    __shared__ __attribute__((aligned(16))) unsigned char smem[LDS_BYTES];
    __shared__ float lds_m[64], lds_l[64];
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63, a = lane >> 4, b = lane & 15;
    LatentTile w;
    if (!find_latent_tile(v, d.heads, blockIdx.x, &w)) return;
    const int ks = d.kp >> 5, rs = d.rp >> 5, kd = d.kp + d.rp, rows = w.q_len * d.heads;
    const int rho = w.tile * 16 + b;
    const bool ok = rho < rows;
    const int tl = ok ? rho / d.heads : 0, h = ok ? rho % d.heads : 0;
    const int row_pos = w.pos0 + tl, win_lo = max(0, row_pos + 1 - d.window);
    const int t_first = w.tile * 16 / d.heads, t_last = min(w.q_len - 1, (w.tile * 16 + 15) / d.heads);
    const int kv_end = w.pos0 + t_last + 1, kv_lo = max(0, w.pos0 + t_first + 1 - d.window);
    const int blk_lo = kv_lo / 16, nblk = (kv_end + 15) / 16 - blk_lo;
    const int per = (nblk + nsplit - 1) / nsplit;
    const int my_lo = blk_lo + (int)blockIdx.y * per, my_hi = min(blk_lo + nblk, my_lo + per);
    const int32_t* bt = v.bt + (long)w.seq * v.max_blocks;

    bf16x8 kf[KS + LATENT_RS], kn[KS + LATENT_RS], qf[KS + LATENT_RS];
    auto load = [&](int blk, bf16x8 (&f)[KS + LATENT_RS]) {
        const bf16* t = p.pool + (long)bt[blk] * 16 * kd + lane * 8;
#pragma unroll
        for (int s = 0; s < KS; s++)
            if (s < ks) f[s] = *reinterpret_cast<const bf16x8*>(t + s * 512);
#pragma unroll
        for (int s = 0; s < LATENT_RS; s++)
            if (s < rs) f[KS + s] = *reinterpret_cast<const bf16x8*>(t + (ks + s) * 512);
    };
    const int first = my_lo + wave;
    if (first < my_hi) load(first, kf);
    {
        const long qrow = (long)(w.tok0 + tl) * d.heads + h;
#pragma unroll
        for (int s = 0; s < KS; s++)
            if (s < ks) qf[s] = *reinterpret_cast<const bf16x8*>(p.q_lat + qrow * d.kp + 32 * s + 8 * a);
#pragma unroll
        for (int s = 0; s < LATENT_RS; s++)
            if (s < rs)
                qf[KS + s] = rotate8(*reinterpret_cast<const bf16x8*>(p.q + qrow * (d.dp + d.rp) + d.dp + 32 * s + 8 * a), 32 * s + 8 * a,
                                     d.rot_dims, p.cos_t, p.sin_t, row_pos);
    }
    bf16* stage = reinterpret_cast<bf16*>(smem) + wave * STAGE;
    // transposed read of d-tile dt: lane i of a 16-lane group names 4 dims of key 4a + i / 4 and receives dim i of keys 4a … 4a + 3
    const int tr_off = ((((lane & 3) >> 1) * 16) + 4 * a + ((lane & 15) >> 2)) * 8 + (lane & 1) * 4;
    float m_run = -INFINITY, l_run = 0.f;
    floatx4 o[DT];
#pragma unroll
    for (int t = 0; t < DT; t++) o[t] = (floatx4){0.f, 0.f, 0.f, 0.f};
    for (int blk = first; blk < my_hi; blk += 4) {
        if (blk + 4 < my_hi) load(blk + 4, kn);
        floatx4 sc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < KS; s++)
            if (s < ks) {
                sc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[s], qf[s], sc, 0, 0, 0);
                *reinterpret_cast<bf16x8*>(stage + s * 512 + lane * 8) = kf[s];
            }
#pragma unroll
        for (int s = 0; s < LATENT_RS; s++)
            if (s < rs) sc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[KS + s], qf[KS + s], sc, 0, 0, 0);
        float mx = -INFINITY;
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const int key = blk * 16 + 4 * a + r;
            sc[r] = ok && key <= row_pos && key >= win_lo ? sc[r] * d.scale : -INFINITY;
            mx = fmaxf(mx, sc[r]);
        }
        const float m_new = fmaxf(m_run, rows_reduce_max(mx)), m_safe = m_new == -INFINITY ? 0.f : m_new;
        const float alpha = __expf(m_run - m_safe);
        float ps = 0.f;
        bf16x4 pf;
#pragma unroll
        for (int r = 0; r < 4; r++) { const float e = __expf(sc[r] - m_safe); ps += e; pf[r] = (bf16)e; }
        l_run = l_run * alpha + rows_reduce_sum(ps);
        m_run = m_new;
#pragma unroll
        for (int t = 0; t < DT; t++)
            if (t < 2 * ks) {
                const shortx4 vt = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) shortx4*)(stage + t * 256 + tr_off));
#pragma unroll
                for (int r = 0; r < 4; r++) o[t][r] *= alpha;
                o[t] = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(vt, __builtin_bit_cast(shortx4, pf), o[t], 0, 0, 0);
            }
#pragma unroll
        for (int s = 0; s < KS + LATENT_RS; s++) kf[s] = kn[s];
    }
    // merge the four waves in wave order: scale by exp(m_w − M), then add into one LDS copy
    if (a == 0) { lds_m[wave * 16 + b] = m_run; lds_l[wave * 16 + b] = l_run; }
    __syncthreads();
    float M = -INFINITY, L = 0.f;
#pragma unroll
    for (int q = 0; q < 4; q++) M = fmaxf(M, lds_m[q * 16 + b]);
    const float Ms = M == -INFINITY ? 0.f : M;
#pragma unroll
    for (int q = 0; q < 4; q++) L += lds_l[q * 16 + b] * __expf(lds_m[q * 16 + b] - Ms);
    const float f = __expf(m_run - Ms);
    float* lo = reinterpret_cast<float*>(smem);
    for (int q = 0; q < 4; q++) {
        if (wave == q) {
#pragma unroll
            for (int t = 0; t < DT; t++)
                if (t < 2 * ks) {
                    floatx4* at = reinterpret_cast<floatx4*>(lo + b * OSTR + t * 16 + 4 * a);
                    floatx4 x = o[t];
#pragma unroll
                    for (int r = 0; r < 4; r++) x[r] *= f;
                    *at = q == 0 ? x : *at + x;
                }
        }
        __syncthreads();
    }
    const int row = threadIdx.x >> 4, c0 = threadIdx.x & 15;      // 16 threads per row
    const float Lr = __shfl(L, row, 64), Mr = __shfl(M, row, 64); // (lane `row` of every wave holds that row's totals)
    if (nsplit > 1) {
        float* dst = p.partial + (((long)blockIdx.x * nsplit + blockIdx.y) * 16 + row) * (d.kp + LATENT_PARTIAL_PAD);
        for (int c = c0 * 4; c < d.kp; c += 64) *reinterpret_cast<floatx4*>(dst + c) = *reinterpret_cast<floatx4*>(lo + row * OSTR + c);
        if (c0 == 0) { dst[d.kp] = Mr; dst[d.kp + 1] = Lr; }
        return;
    }
    const int ro = w.tile * 16 + row;
    if (ro >= rows) return;
    const float inv = Lr > 0.f ? 1.0f / Lr : 0.f;
    bf16* dst = p.o_lat + ((long)w.tok0 * d.heads + ro) * d.kp;
    for (int c = c0 * 4; c < d.kp; c += 64) {
        const floatx4 x = *reinterpret_cast<floatx4*>(lo + row * OSTR + c);
        bf16x4 y;
#pragma unroll
        for (int r = 0; r < 4; r++) y[r] = (bf16)(x[r] * inv);
        *reinterpret_cast<bf16x4*>(dst + c) = y;
    }
}
// one workgroup per row tile, 16 threads per row
__global__ __launch_bounds__(256) void latent_attn_reduce_kernel(LatentDims d, LatentBuffers<bf16> p, BatchView v, int nsplit) {
    LatentTile w;
    if (!find_latent_tile(v, d.heads, blockIdx.x, &w)) return;
    const int row = threadIdx.x >> 4, c0 = threadIdx.x & 15, ro = w.tile * 16 + row;
    if (ro >= w.q_len * d.heads) return;
    const long ld = d.kp + LATENT_PARTIAL_PAD;
    const float* src = p.partial + ((long)blockIdx.x * nsplit * 16 + row) * ld;
    float M = -INFINITY, L = 0.f;
    for (int z = 0; z < nsplit; z++) M = fmaxf(M, src[z * 16 * ld + d.kp]);
    for (int z = 0; z < nsplit; z++) L += src[z * 16 * ld + d.kp + 1] * __expf(src[z * 16 * ld + d.kp] - M);
    const float inv = 1.0f / L;
    for (int c = c0 * 4; c < d.kp; c += 64) {
        floatx4 acc = {0.f, 0.f, 0.f, 0.f};
        for (int z = 0; z < nsplit; z++) acc += *reinterpret_cast<const floatx4*>(src + z * 16 * ld + c) * (__expf(src[z * 16 * ld + d.kp] - M) * inv);
        bf16x4 y;
#pragma unroll
        for (int r = 0; r < 4; r++) y[r] = (bf16)acc[r];
        *reinterpret_cast<bf16x4*>(p.o_lat + ((long)w.tok0 * d.heads + ro) * d.kp + c) = y;
    }
}

template <typename E>
static int latent_plain(const LatentDims& d, const LatentBuffers<E>& b, const BatchView& v, hipStream_t s) {
    form_hit(FORM_LATENT_ATTN_PLAIN);
    const size_t lds = (size_t)(2 * d.kp + d.rp + 256 + 8) * 4;
    FH_REQUIRE(lds <= 64 * 1024, "latent attention: kv_rank %d + rotated %d do not fit LDS", d.kv_rank, d.rot_dim);
    hipLaunchKernelGGL(latent_attn_plain_kernel<E>, dim3(v.T, d.heads), dim3(256), lds, s, d, b, v);
    FH_CHECK_LAUNCH();
    return 0;
}
static int latent_mfma(const LatentDims& d, const LatentBuffers<bf16>& b, const BatchView& v, hipStream_t s) {
    const int tiles = (int)(((long)v.T * d.heads) / 16) + v.num_seqs;      // upper bound of Σ ceil(rows / 16)
    const int keys = std::min(v.max_keys, d.window + 16);
    // split the keys while the launch has fewer than ≈ 2 workgroups per CU and a split keeps ≥ 128 keys (two blocks per wave)
    int ns = 1;
    while (ns < 16 && tiles * ns < 256 && keys >= 2 * ns * 128) ns *= 2;
    if (knobs().latent_splits > 0) ns = std::min(16, knobs().latent_splits);
    while (ns > 1 && (size_t)tiles * ns * 16 * (d.kp + LATENT_PARTIAL_PAD) * 4 > b.partial_bytes) ns /= 2;
    const dim3 grid(tiles, ns);
    form_hit(ns > 1 ? FORM_LATENT_ATTN_SPLIT : FORM_LATENT_ATTN);
    if (d.kp <= 64) hipLaunchKernelGGL(latent_attn_kernel<2>, grid, dim3(256), 0, s, d, b, v, ns);
    else if (d.kp <= 128) hipLaunchKernelGGL(latent_attn_kernel<4>, grid, dim3(256), 0, s, d, b, v, ns);
    else if (d.kp <= 256) hipLaunchKernelGGL(latent_attn_kernel<8>, grid, dim3(256), 0, s, d, b, v, ns);
    else hipLaunchKernelGGL(latent_attn_kernel<16>, grid, dim3(256), 0, s, d, b, v, ns);
    FH_CHECK_LAUNCH();
    if (ns > 1) {
        hipLaunchKernelGGL(latent_attn_reduce_kernel, dim3(tiles), dim3(256), 0, s, d, b, v, ns);
        FH_CHECK_LAUNCH();
    }
    return 0;
}
template <> int latent_attention<float>(const LatentDims& d, const LatentBuffers<float>& b, const BatchView& v, hipStream_t s) {
    return latent_plain(d, b, v, s);
}
template <> int latent_attention<bf16>(const LatentDims& d, const LatentBuffers<bf16>& b, const BatchView& v, hipStream_t s) {
    if (knobs().latent_plain || d.kp > 512 || d.rp > 32 * LATENT_RS) return latent_plain(d, b, v, s);
    return latent_mfma(d, b, v, s);
}
template int latent_prepare<bf16>(const bf16*, const bf16*, long, const float*, const float*, float, const LatentDims&, const LatentBuffers<bf16>&,
                                  const BatchView&, bf16*, hipStream_t);
template int latent_prepare<float>(const float*, const float*, long, const float*, const float*, float, const LatentDims&,
                                   const LatentBuffers<float>&, const BatchView&, float*, hipStream_t);

}  // namespace fh
