// Dense projections over weights stored as MFMA-fragment tiles, for 16-bit and 32-bit models.
//
// Tile layout (the one f16t uses): [groups][n / 16][k / 32][64 lanes][8]; lane (a, b) of a k-step holds W[16·tile + b][32·step + 8a .. +8],
// so a wave load of a fragment is contiguous and IS the B operand.  The 32-bit form keeps the same 8 values per lane and feeds them
// to eight v_mfma_f32_16x16x4_f32: both operands permute the contraction index the same way, so no re-layout is needed.
// n and k are padded to multiples of 32 with zero rows / columns, activations have padded leading dimensions: no kernel masks K.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

namespace fh {

typedef __bf16 bf16;
typedef bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef bf16 bf16x4 __attribute__((ext_vector_type(4)));
typedef float floatx8 __attribute__((ext_vector_type(8)));
typedef float floatx4 __attribute__((ext_vector_type(4)));
typedef short shortx4 __attribute__((ext_vector_type(4)));

template <typename E> struct Frag;
template <> struct Frag<bf16> {
    typedef bf16x8 v8;
    static __device__ __forceinline__ floatx4 mma(v8 a, v8 b, floatx4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }
};
template <> struct Frag<float> {
    typedef floatx8 v8;
    static __device__ __forceinline__ floatx4 mma(v8 a, v8 b, floatx4 c) {
#pragma unroll
        for (int j = 0; j < 8; j++) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[j], b[j], c, 0, 0, 0);
        return c;
    }
};

static inline int pad32(int n) { return (n + 31) / 32 * 32; }

enum GemmAct : int { GEMM_ACT_NONE = 0, GEMM_ACT_SIGMOID = 1, GEMM_ACT_GELU_TANH = 2, GEMM_ACT_XIELU = 3, GEMM_ACT_RELU2 = 4, GEMM_ACT_CLAMPED_GLU = 5,
                     GEMM_ACT_SILU_GLU = 6, GEMM_ACT_GELU_GLU = 7, GEMM_ACT_SILU = 8, GEMM_ACT_SOFTPLUS = 9, GEMM_ACT_LOG_SIGMOID = 10,
                     GEMM_ACT_SOFTCAP = 11 };
// sections of (gate, up) pairs
__host__ __device__ inline bool gemm_gated_act(int act) { return act >= GEMM_ACT_CLAMPED_GLU && act <= GEMM_ACT_GELU_GLU; }
// inputs of a recurrence and capped logits, a launch form of their own
__host__ __device__ inline bool gemm_rare_act(int act) { return act >= GEMM_ACT_SOFTPLUS; }
constexpr int GEMM_MAX_SECTIONS = 6;
struct GemmSection {          // columns [begin, next section's begin) of a fused projection; begin is a multiple of 32
    int begin, act;
    float p, q;               // xIELU: softplus of its two parameters; clamped GLU: limit, slope of the sigmoid; log σ: factor p; softcap: cap p
    float mul = 1.f;          // factor of the accumulator, ahead of bias and activation (a norm's gain that is a single number)
};
// A gated section pairs 16-column tiles (gate, up, gate, up, …) whose weights are packed that way; a wave holds both tiles of a pair, and
// the result takes the first half of the section's columns.

// Rows sorted by weight group (an expert's tokens), in blocks of `block` rows of one group each; the kernels read the block count from
// the device, so a launch is sized for the largest one.  Place p of the list stands for row id[p] of the output and row id[p] / div of x;
// ids of m and more are padding.
struct GemmRows {
    const int32_t *id = nullptr, *group = nullptr, *total = nullptr;      // [places], [blocks], places in use
    int block = 0, max_blocks = 0, div = 1;
};

// out[r][g·out_group + c] = act(mul · x[r][g·x_group ..] · W_gᵀ + bias) · row_scale[r][g] · col_scale[col_scale_row[r]][c]
template <typename E>
struct TiledGemm {
    const E* x = nullptr; long ldx = 0, x_group = 0;
    // rows from a cache of 16-row fragment blocks instead ([k / 8][16 rows][8] each): row tile i is block x_blocks[i] of x
    const int32_t* x_blocks = nullptr; long x_block_elems = 0;
    const E* w = nullptr;
    const float* bias = nullptr;          // [groups·n]
    int m = 0, n = 0, k = 0, groups = 1;
    int n_store = 0;                      // columns written (0: all n)
    E* out = nullptr; float* out_f32 = nullptr;      // one of the two
    long ldo = 0, out_group = 0;
    int slabs = 1; long slab_stride = 0;  // > 1: K split over workgroups, part z at out_f32 + z·slab_stride, summed by the consumer
    const E* row_scale = nullptr; long ld_scale = 0;
    const E* col_scale = nullptr; const uint32_t* col_scale_row = nullptr; long ld_col_scale = 0;
    GemmRows rows;                        // (bias, groups and the x / out group strides are not used with it)
    int nsec = 0;
    GemmSection sec[GEMM_MAX_SECTIONS] = {};
};
template <typename E> int tiled_gemm(const TiledGemm<E>& g, hipStream_t s);
// number of K parts worth making for a projection of m rows whose consumer sums slabs (≤ GEMM_MAX_SLABS)
constexpr int GEMM_MAX_SLABS = 8;
int tiled_gemm_slabs(int m, int n, int k);

// Activations on fp32 accumulators.  Models in 16 bits round the result to 2⁻⁹, so their form uses the hardware exponential and
// reciprocal (relative error ≈ 2⁻²²); 32-bit models call the library functions.
template <typename E> struct ActMath;
template <> struct ActMath<float> {
    static __device__ __forceinline__ float sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
    static __device__ __forceinline__ float tanh(float z) { return tanhf(z); }
    static __device__ __forceinline__ float expm1_minus(float z) { return expm1f(z) - z; }
    static __device__ __forceinline__ float log1p_exp_minus(float z) { return log1pf(expf(-z)); }
};
template <> struct ActMath<bf16> {
    static __device__ __forceinline__ float sigmoid(float z) { return __builtin_amdgcn_rcpf(1.0f + __expf(-z)); }
    static __device__ __forceinline__ float tanh(float z) { return 1.0f - 2.0f * __builtin_amdgcn_rcpf(1.0f + __expf(2.0f * z)); }
    static __device__ __forceinline__ float expm1_minus(float z) { return __expf(z) - 1.0f - z; }
    // to fp32 rounding: the logarithm of the rounded 1 + e, corrected by the ratio of e to what was added (Kahan)
    static __device__ __forceinline__ float log1p_exp_minus(float z) {
        const float e = __expf(-z), u = 1.0f + e, added = u - 1.0f;
        return added > 0.f ? __logf(u) * (e * __builtin_amdgcn_rcpf(added)) : e;
    }
};
template <typename E>
__device__ __forceinline__ float gelu_tanh_f32(float z) {
    return 0.5f * z * (1.0f + ActMath<E>::tanh(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}
// gate bounded from above, linear half on both sides
template <typename E>
__device__ __forceinline__ float clamped_glu_f32(float g, float u, float limit, float slope) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g * ActMath<E>::sigmoid(slope * g) * (u + 1.0f);
}
// inputs of a recurrence, to fp32 rounding in both number formats
template <typename E>
__device__ __forceinline__ float softplus_f32(float z) { return fmaxf(z, 0.f) + ActMath<E>::log1p_exp_minus(fabsf(z)); }
template <typename E>
__device__ __forceinline__ float log_sigmoid_f32(float z) { return fminf(z, 0.f) - ActMath<E>::log1p_exp_minus(fabsf(z)); }
// quadratic right of zero, exponential left of it, slope 1/2 at zero; sp / sq: softplus of the two trained numbers
template <typename E>
__device__ __forceinline__ float xielu_f32(float z, float sp, float sq) {
    return (z > 0.f ? sp * z * z : (0.5f + sq) * ActMath<E>::expm1_minus(z)) + 0.5f * z;
}

}  // namespace fh
