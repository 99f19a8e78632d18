// Residual stream of the layered models: fp32 throughout, with a copy in the projections' number format written by whoever changes it.
#include "common.h"
#include "layer_ops.h"

namespace fh {

template <typename E, bool VEC>
__global__ __launch_bounds__(256) void embed_kernel(Embedding<E> p, BatchView v, float* __restrict__ x, E* __restrict__ xb, int dim, int ldb) {
    const int t = blockIdx.x;
    const uint32_t tok = v.tokens[t];
    const E *own = p.table + (long)tok * dim, *bigram = nullptr, *place = nullptr;
    if (p.bigram || p.positions) {
        const int seq = v.tok_seq[t], at = t - (int)v.cu[seq];
        if (p.bigram) {
            const int64_t prev = at == 0 ? (int64_t)v.prev[seq] : (int64_t)v.tokens[t - 1];
            bigram = p.bigram + dim * (prev < 0 ? (long)p.buckets : (long)(((uint64_t)prev * (uint64_t)p.mul_prev + (uint64_t)tok * (uint64_t)p.mul_cur) % (uint64_t)p.buckets));
        }
        if (p.positions) place = p.positions + (long)(v.pos[seq] + at) * dim;
    }
    if (VEC) {
        typedef typename Frag<E>::v8 v8;
        for (int i = threadIdx.x * 8; i < dim; i += 2048) {
            const v8 e = *reinterpret_cast<const v8*>(own + i);
            v8 g = e, l = e, o;
            if (bigram) g = *reinterpret_cast<const v8*>(bigram + i);
            if (place) l = *reinterpret_cast<const v8*>(place + i);
            floatx4 f[2];
#pragma unroll
            for (int j = 0; j < 8; j++) {
                const float y = (float)e[j] * p.factor + (bigram ? (float)g[j] : 0.f) + (place ? (float)l[j] : 0.f);
                f[j >> 2][j & 3] = y;
                o[j] = (E)y;
            }
            *reinterpret_cast<floatx4*>(x + (long)t * dim + i) = f[0];
            *reinterpret_cast<floatx4*>(x + (long)t * dim + i + 4) = f[1];
            *reinterpret_cast<v8*>(xb + (long)t * ldb + i) = o;
        }
        return;
    }
    for (int i = threadIdx.x; i < dim; i += 256) {
        float e = (float)own[i] * p.factor;
        if (bigram) e += (float)bigram[i];
        if (place) e += (float)place[i];
        x[(long)t * dim + i] = e;
        xb[(long)t * ldb + i] = (E)e;
    }
}

template <typename E>
int embed_tokens(const Embedding<E>& e, const BatchView& v, float* x, E* xb, int dim, int ldb, hipStream_t s) {
    if (dim % 8 == 0) hipLaunchKernelGGL((embed_kernel<E, true>), dim3(v.T), dim3(256), 0, s, e, v, x, xb, dim, ldb);
    else hipLaunchKernelGGL((embed_kernel<E, false>), dim3(v.T), dim3(256), 0, s, e, v, x, xb, dim, ldb);
    FH_CHECK_LAUNCH();
    return 0;
}

__device__ __forceinline__ float block_sum(float q, float* red) {
    q = wave_reduce_sum(q);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = q;
    __syncthreads();
    float t = 0.f;
    for (int i = 0; i < (int)(blockDim.x >> 6); i++) t += red[i];
    return t;
}

// x += Σ slabs of `sub` + Σ_j weights[row][j] · pairs[row·top + j]; elementwise, grid (rows, quads of columns / 256)
template <typename E, bool VEC>
__global__ __launch_bounds__(256) void branch_add_kernel(const float* __restrict__ sub, long ld_sub, int slabs, long slab_stride, const E* __restrict__ pairs,
                                                         long ld_pair, const float* __restrict__ weights, int top, float* __restrict__ x,
                                                         E* __restrict__ xb, int dim, int ldb) {
    const long row = blockIdx.x;
    const int i = (blockIdx.y * 256 + threadIdx.x) * 4;
    if (i >= dim) return;
    const float* sr = sub + row * ld_sub + i;
    const E* pr = pairs + row * top * ld_pair + i;
    if (VEC) {
        typedef E e4 __attribute__((ext_vector_type(4)));
        floatx4 v = *reinterpret_cast<const floatx4*>(sr);
        const floatx4 xv = *reinterpret_cast<const floatx4*>(x + row * dim + i);
        for (int z = 1; z < slabs; z++) v += *reinterpret_cast<const floatx4*>(sr + z * slab_stride);
#pragma unroll 4
        for (int j = 0; j < top; j++) {
            const e4 e = *reinterpret_cast<const e4*>(pr + j * ld_pair);
            const float w = weights[row * top + j];
#pragma unroll
            for (int k = 0; k < 4; k++) v[k] += w * (float)e[k];
        }
        v += xv;
        e4 o;
#pragma unroll
        for (int k = 0; k < 4; k++) o[k] = (E)v[k];
        *reinterpret_cast<floatx4*>(x + row * dim + i) = v;
        *reinterpret_cast<e4*>(xb + row * ldb + i) = o;
        return;
    }
    for (int k = 0; k < 4 && i + k < dim; k++) {
        float v = sr[k];
        for (int z = 1; z < slabs; z++) v += sr[z * slab_stride + k];
        for (int j = 0; j < top; j++) v += weights[row * top + j] * (float)pr[j * ld_pair + k];
        v += x[row * dim + i + k];
        x[row * dim + i + k] = v;
        xb[row * ldb + i + k] = (E)v;
    }
}
template <typename E>
int branch_add(const float* sub, long ld_sub, int slabs, long slab_stride, const E* pairs, long ld_pair, const float* weights, int top, float* x, E* xb,
               int rows, int dim, int ldb, hipStream_t s) {
    const bool vec = dim % 4 == 0 && ld_sub % 4 == 0 && ld_pair % 4 == 0 && ldb % 4 == 0 && slab_stride % 4 == 0;
    const dim3 grid(rows, cdiv(dim, 1024));
    if (vec) hipLaunchKernelGGL((branch_add_kernel<E, true>), grid, dim3(256), 0, s, sub, ld_sub, slabs, slab_stride, pairs, ld_pair, weights, top, x, xb, dim, ldb);
    else hipLaunchKernelGGL((branch_add_kernel<E, false>), grid, dim3(256), 0, s, sub, ld_sub, slabs, slab_stride, pairs, ld_pair, weights, top, x, xb, dim, ldb);
    FH_CHECK_LAUNCH();
    return 0;
}

// One workgroup per row; a thread holds up to 4 quads of the row in registers, so the branch is read once.  NEXT: the copy is the row
// divided by its root mean square, the input of a block that norms ahead of its sublayers.
template <typename E, bool VEC, bool GATE, bool NEXT>
__global__ __launch_bounds__(1024) void post_norm_add_kernel(const float* __restrict__ sub, long ld_sub, int slabs, long slab_stride, const E* __restrict__ gate,
                                                             long ld_gate, const float* __restrict__ w, float mult, float eps,
                                                             float* __restrict__ x, E* __restrict__ xb, int dim, int ldb) {
    __shared__ float red[32];
    const long row = blockIdx.x;
    const float* sr = sub + row * ld_sub;
    const E* gr = GATE ? gate + row * ld_gate : nullptr;
    float* xr = x + row * dim;
    E* br = xb + row * ldb;
    float q = 0.f, n = 0.f;
    if (VEC) {
        typedef E e4 __attribute__((ext_vector_type(4)));
        floatx4 v[4], xv[4], wv[4];
#pragma unroll
        for (int c = 0; c < 4; c++) {
            const int i = (c * blockDim.x + threadIdx.x) * 4;
            if (i < dim) {
                v[c] = *reinterpret_cast<const floatx4*>(sr + i);
                for (int z = 1; z < slabs; z++) v[c] += *reinterpret_cast<const floatx4*>(sr + z * slab_stride + i);
                e4 gv = {};
                if (GATE) gv = *reinterpret_cast<const e4*>(gr + i);
                xv[c] = *reinterpret_cast<const floatx4*>(xr + i);
                wv[c] = *reinterpret_cast<const floatx4*>(w + i);
#pragma unroll
                for (int j = 0; j < 4; j++) { if (GATE) v[c][j] *= (float)gv[j]; q += v[c][j] * v[c][j]; }
            }
        }
        const float inv = mult / sqrtf(block_sum(q, red) / (float)dim + eps);
#pragma unroll
        for (int c = 0; c < 4; c++) {
            const int i = (c * blockDim.x + threadIdx.x) * 4;
            if (i < dim) {
#pragma unroll
                for (int j = 0; j < 4; j++) { xv[c][j] += v[c][j] * inv * wv[c][j]; n += xv[c][j] * xv[c][j]; }
                *reinterpret_cast<floatx4*>(xr + i) = xv[c];
            }
        }
        const float unit = NEXT ? 1.0f / sqrtf(block_sum(n, red + 16) / (float)dim + eps) : 1.0f;
#pragma unroll
        for (int c = 0; c < 4; c++) {
            const int i = (c * blockDim.x + threadIdx.x) * 4;
            if (i < dim) {
                e4 o;
#pragma unroll
                for (int j = 0; j < 4; j++) o[j] = (E)(xv[c][j] * unit);
                *reinterpret_cast<e4*>(br + i) = o;
            }
        }
        return;
    }
    auto branch = [&](int i) {
        float t = sr[i];
        for (int z = 1; z < slabs; z++) t += sr[z * slab_stride + i];
        return GATE ? t * (float)gr[i] : t;
    };
    for (int i = threadIdx.x; i < dim; i += blockDim.x) { const float t = branch(i); q += t * t; }
    const float inv = mult / sqrtf(block_sum(q, red) / (float)dim + eps);
    for (int i = threadIdx.x; i < dim; i += blockDim.x) {
        const float t = xr[i] + branch(i) * inv * w[i];
        xr[i] = t;
        n += t * t;
        if (!NEXT) br[i] = (E)t;
    }
    if (NEXT) {
        const float unit = 1.0f / sqrtf(block_sum(n, red + 16) / (float)dim + eps);
        for (int i = threadIdx.x; i < dim; i += blockDim.x) br[i] = (E)(xr[i] * unit);
    }
}

template <typename E>
int post_norm_add(const float* sub, long ld_sub, int slabs, long slab_stride, const E* gate, long ld_gate, const float* w, float mult, float eps, bool next_norm,
                  float* x, E* xb, int rows, int dim, int ldb, hipStream_t s) {
    const int threads = rows <= 512 && dim >= 2048 ? 1024 : 256;
    const bool vec = dim % 4 == 0 && dim <= threads * 16 && ld_sub % 4 == 0 && ld_gate % 4 == 0 && ldb % 4 == 0 && slab_stride % 4 == 0;
#define POST(V, G, N) hipLaunchKernelGGL((post_norm_add_kernel<E, V, G, N>), dim3(rows), dim3(threads), 0, s, sub, ld_sub, slabs, slab_stride, gate, ld_gate, w, mult, eps, x, xb, dim, ldb)
    if (gate) { if (next_norm) { if (vec) POST(true, true, true); else POST(false, true, true); } else { if (vec) POST(true, true, false); else POST(false, true, false); } }
    else { if (next_norm) { if (vec) POST(true, false, true); else POST(false, false, true); } else { if (vec) POST(true, false, false); else POST(false, false, false); } }
#undef POST
    FH_CHECK_LAUNCH();
    return 0;
}

template <typename E>
__global__ __launch_bounds__(256) void copy_rows_kernel(const E* __restrict__ x, long ldx, E* __restrict__ out, long ldo, int cols) {
    for (int i = threadIdx.x; i < cols; i += 256) out[blockIdx.x * ldo + i] = x[blockIdx.x * ldx + i];
}
template <typename E>
int copy_rows(const E* x, long ldx, E* out, long ldo, int rows, int cols, hipStream_t s) {
    hipLaunchKernelGGL(copy_rows_kernel<E>, dim3(rows), dim3(256), 0, s, x, ldx, out, ldo, cols);
    FH_CHECK_LAUNCH();
    return 0;
}

template <typename E>
__global__ __launch_bounds__(256) void rms_norm_rows_kernel(const float* __restrict__ x, const int32_t* __restrict__ row_idx,
                                                            const float* __restrict__ w, float eps, E* __restrict__ out, int dim, int ldo) {
    __shared__ float red[4];
    const float* xr = x + (row_idx ? (long)row_idx[blockIdx.x] : (long)blockIdx.x) * dim;
    float q = 0.f;
    for (int i = threadIdx.x; i < dim; i += 256) q += xr[i] * xr[i];
    const float inv = 1.0f / sqrtf(block_sum(q, red) / (float)dim + eps);
    for (int i = threadIdx.x; i < dim; i += 256) out[(long)blockIdx.x * ldo + i] = (E)(w ? xr[i] * inv * w[i] : xr[i] * inv);
}
template <typename E>
int rms_norm_rows(const float* x, const int32_t* row_idx, const float* w, float eps, E* out, int rows, int dim, int ldo, hipStream_t s) {
    hipLaunchKernelGGL(rms_norm_rows_kernel<E>, dim3(rows), dim3(256), 0, s, x, row_idx, w, eps, out, dim, ldo);
    FH_CHECK_LAUNCH();
    return 0;
}

// One workgroup per row; a thread holds up to 4 quads of the row in registers.  POST: the sum itself is normed.
template <typename E, bool VEC, bool POST>
__global__ __launch_bounds__(1024) void stream_update_kernel(StreamUpdate<E> u) {
    __shared__ float red[64];
    const long row = blockIdx.x;
    const int dim = u.dim, nt = blockDim.x;
    const float *s1 = u.sub + row * u.ld_sub, *s2 = u.sub2 + row * u.ld_sub;
    float* xr = u.x + row * dim;
    const E* pr = u.pairs + row * u.top * u.ld_pair;
    E* out = u.out + row * u.ldo;
    const bool joined = !POST && u.sub2 != nullptr;
    float keep = u.replace ? 0.f : 1.f, factor = 1.f;
    if (POST) {
        keep *= u.keep;
        if (u.sub_scale) factor = u.sub_scale[row];
        if (u.pair_ids)
            for (int j = 0; j < u.top; j++)
                if (u.pair_ids[row * u.top + j] >= u.pair_limit) keep += u.weights[row * u.top + j];
    }
    auto listed = [&](int j) { return !POST || !u.pair_ids || u.pair_ids[row * u.top + j] < u.pair_limit; };
    if (VEC) {
        typedef E e4 __attribute__((ext_vector_type(4)));
        floatx4 v[4], r[4], xv[4];
        float q1 = 0.f, q2 = 0.f, n = 0.f;
#pragma unroll
        for (int c = 0; c < 4; c++) {
            const int i = (c * nt + threadIdx.x) * 4;
            if (i < dim) {
                v[c] = (floatx4){0.f, 0.f, 0.f, 0.f};
                if (u.sub) v[c] = *reinterpret_cast<const floatx4*>(s1 + i);
                for (int z = 1; z < u.slabs; z++) v[c] += *reinterpret_cast<const floatx4*>(s1 + z * u.slab_stride + i);
                if (POST)
#pragma unroll
                    for (int k = 0; k < 4; k++) v[c][k] *= factor;
                xv[c] = (floatx4){0.f, 0.f, 0.f, 0.f};
                if (!u.replace) xv[c] = *reinterpret_cast<const floatx4*>(xr + i);
                if (POST)
#pragma unroll
                    for (int k = 0; k < 4; k++) xv[c][k] *= keep;
                if (u.add) xv[c] += *reinterpret_cast<const floatx4*>(u.add + i);
#pragma unroll 4
                for (int j = 0; j < u.top; j++) {
                    if (!listed(j)) continue;
                    const e4 e = *reinterpret_cast<const e4*>(pr + j * u.ld_pair + i);
                    const float w = u.weights[row * u.top + j];
#pragma unroll
                    for (int k = 0; k < 4; k++) v[c][k] += w * (float)e[k];
                }
                if (joined) {
                    r[c] = *reinterpret_cast<const floatx4*>(s2 + i);
                    for (int z = 1; z < u.slabs2; z++) r[c] += *reinterpret_cast<const floatx4*>(s2 + z * u.slab_stride2 + i);
#pragma unroll
                    for (int k = 0; k < 4; k++) { q1 += v[c][k] * v[c][k]; q2 += r[c][k] * r[c][k]; }
                }
            }
        }
        float i1 = 0.f, i2 = 0.f;
        if (joined) {
            i1 = 0.5f / sqrtf(block_sum(q1, red) / (float)dim + u.eps);
            i2 = 0.5f / sqrtf(block_sum(q2, red + 16) / (float)dim + u.eps);
        }
#pragma unroll
        for (int c = 0; c < 4; c++) {
            const int i = (c * nt + threadIdx.x) * 4;
            if (i < dim) {
                if (joined) {
                    const floatx4 w1 = *reinterpret_cast<const floatx4*>(u.w + i), w2 = *reinterpret_cast<const floatx4*>(u.w2 + i);
#pragma unroll
                    for (int k = 0; k < 4; k++) v[c][k] = v[c][k] * i1 * w1[k] + r[c][k] * i2 * w2[k];
                }
                xv[c] += v[c];
#pragma unroll
                for (int k = 0; k < 4; k++) n += xv[c][k] * xv[c][k];
                if (!POST) *reinterpret_cast<floatx4*>(xr + i) = xv[c];
            }
        }
        if (POST) {
            const float inv = 1.0f / sqrtf(block_sum(n, red) / (float)dim + u.eps);
            float z = 0.f;
            n = 0.f;
#pragma unroll
            for (int c = 0; c < 4; c++) {
                const int i = (c * nt + threadIdx.x) * 4;
                if (i < dim) {
                    const floatx4 w = *reinterpret_cast<const floatx4*>(u.post_w + i);
                    floatx4 g = {0.f, 0.f, 0.f, 0.f};
                    if (u.gate) g = *reinterpret_cast<const floatx4*>(u.gate_w + i);
#pragma unroll
                    for (int k = 0; k < 4; k++) { xv[c][k] *= inv * w[k]; n += xv[c][k] * xv[c][k]; z += xv[c][k] * g[k]; }
                    *reinterpret_cast<floatx4*>(xr + i) = xv[c];
                }
            }
            if (u.gate) {
                z = block_sum(z, red + 16);
                if (threadIdx.x == 0) u.gate[row] = 1.0f / (1.0f + expf(-z));
            }
        }
        if (!u.out) return;
        const float unit = u.next_w ? 1.0f / sqrtf(block_sum(n, red + 32) / (float)dim + u.eps) : 1.0f;
#pragma unroll
        for (int c = 0; c < 4; c++) {
            const int i = (c * nt + threadIdx.x) * 4;
            if (i < dim) {
                floatx4 w = {1.f, 1.f, 1.f, 1.f};
                if (u.next_w) w = *reinterpret_cast<const floatx4*>(u.next_w + i);
                e4 o;
#pragma unroll
                for (int k = 0; k < 4; k++) o[k] = (E)(xv[c][k] * unit * w[k]);
                *reinterpret_cast<e4*>(out + i) = o;
            }
        }
        return;
    }
    auto first = [&](int i) {
        float t = u.sub ? s1[i] : 0.f;
        for (int z = 1; z < u.slabs; z++) t += s1[z * u.slab_stride + i];
        t *= factor;
        for (int j = 0; j < u.top; j++)
            if (listed(j)) t += u.weights[row * u.top + j] * (float)pr[j * u.ld_pair + i];
        return t;
    };
    auto second = [&](int i) {
        float t = s2[i];
        for (int z = 1; z < u.slabs2; z++) t += s2[z * u.slab_stride2 + i];
        return t;
    };
    float i1 = 0.f, i2 = 0.f, n = 0.f;
    if (joined) {
        float q1 = 0.f, q2 = 0.f;
        for (int i = threadIdx.x; i < dim; i += nt) { const float a = first(i), b = second(i); q1 += a * a; q2 += b * b; }
        i1 = 0.5f / sqrtf(block_sum(q1, red) / (float)dim + u.eps);
        i2 = 0.5f / sqrtf(block_sum(q2, red + 16) / (float)dim + u.eps);
    }
    for (int i = threadIdx.x; i < dim; i += nt) {
        float t = joined ? first(i) * i1 * u.w[i] + second(i) * i2 * u.w2[i] : first(i);
        if (u.add) t += u.add[i];
        if (!u.replace) t += POST ? keep * xr[i] : xr[i];
        xr[i] = t;
        n += t * t;
    }
    if (POST) {
        const float inv = 1.0f / sqrtf(block_sum(n, red) / (float)dim + u.eps);
        float z = 0.f;
        n = 0.f;
        for (int i = threadIdx.x; i < dim; i += nt) {            // (a thread's own elements)
            const float t = xr[i] * inv * u.post_w[i];
            xr[i] = t;
            n += t * t;
            if (u.gate) z += t * u.gate_w[i];
        }
        if (u.gate) {
            z = block_sum(z, red + 16);
            if (threadIdx.x == 0) u.gate[row] = 1.0f / (1.0f + expf(-z));
        }
    }
    if (!u.out) return;
    const float unit = u.next_w ? 1.0f / sqrtf(block_sum(n, red + 32) / (float)dim + u.eps) : 1.0f;
    for (int i = threadIdx.x; i < dim; i += nt) out[i] = (E)(u.next_w ? xr[i] * unit * u.next_w[i] : xr[i]);
}
template <typename E>
int stream_update(const StreamUpdate<E>& u, hipStream_t s) {
    FH_REQUIRE(!u.sub2 || (u.sub && u.w && u.w2 && !u.top), "stream update: a second branch needs both norms");
    FH_REQUIRE(u.sub || u.slabs == 1, "stream update: slabs of nothing");
    FH_REQUIRE(u.post_w ? !u.sub2 : u.keep == 1.f && !u.pair_ids && !u.sub_scale && !u.gate, "stream update: factors and the stream's own pairs belong to a normed sum of one branch");
    const int threads = u.rows <= 512 && u.dim >= 2048 ? 1024 : 256;
    const bool vec = u.dim % 4 == 0 && u.dim <= threads * 16 && u.ld_sub % 4 == 0 && u.ld_pair % 4 == 0 && u.ldo % 4 == 0 && u.slab_stride % 4 == 0 && u.slab_stride2 % 4 == 0;
#define UPDATE(V, P) hipLaunchKernelGGL((stream_update_kernel<E, V, P>), dim3(u.rows), dim3(threads), 0, s, u)
    if (u.post_w) { if (vec) UPDATE(true, true); else UPDATE(false, true); }
    else { if (vec) UPDATE(true, false); else UPDATE(false, false); }
#undef UPDATE
    FH_CHECK_LAUNCH();
    return 0;
}

#define INSTANTIATE(E)                                                                                                                  \
    template int embed_tokens<E>(const Embedding<E>&, const BatchView&, float*, E*, int, int, hipStream_t);                              \
    template int branch_add<E>(const float*, long, int, long, const E*, long, const float*, int, float*, E*, int, int, int, hipStream_t); \
    template int post_norm_add<E>(const float*, long, int, long, const E*, long, const float*, float, float, bool, float*, E*, int, int, \
                                  int, hipStream_t);                                                                                    \
    template int copy_rows<E>(const E*, long, E*, long, int, int, hipStream_t);                                                          \
    template int stream_update<E>(const StreamUpdate<E>&, hipStream_t);                                                                  \
    template int rms_norm_rows<E>(const float*, const int32_t*, const float*, float, E*, int, int, int, hipStream_t);
INSTANTIATE(bf16)
INSTANTIATE(float)
#undef INSTANTIATE

}  // namespace fh
