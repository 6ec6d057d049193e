// Interfaces between the block-decoder runtime (blocks.hip) and its kernels (dense_gemv.hip, dense_gemm.hip,
// mixer_attention.hip).  Host side; not part of the C ABI.
#pragma once
#include "ptm_common.h"

namespace ptm {

inline int up8(int n) { return (n + 7) & ~7; }
inline int up64(int n) { return (n + 63) & ~63; }

__device__ __forceinline__ float bf16_lo(uint32_t u) { return __uint_as_float(u << 16); }
__device__ __forceinline__ float bf16_hi(uint32_t u) { return __uint_as_float(u & 0xffff0000u); }
__device__ __forceinline__ float bf16_f(uint16_t u) { return __uint_as_float((uint32_t)u << 16); }
__device__ __forceinline__ uint16_t f_bf16(float f) { return __builtin_bit_cast(uint16_t, (__bf16)f); }  // nearest even

// element access of an activation / cache buffer: bfloat16 or fp32
template <bool F32>
__device__ __forceinline__ void put_elem(void* p, int64_t i, float v) {
    if constexpr (F32) static_cast<float*>(p)[i] = v;
    else static_cast<uint16_t*>(p)[i] = f_bf16(v);
}
template <bool F32>
__device__ __forceinline__ float get_elem(const void* p, int64_t i) {
    if constexpr (F32) return static_cast<const float*>(p)[i];
    else return bf16_f(static_cast<const uint16_t*>(p)[i]);
}

__device__ __forceinline__ float gelu_tanh(float z) {
    return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

// block-wide sum for WAVES waves; red: WAVES floats of LDS
template <int WAVES>
__device__ __forceinline__ float block_sum(float v, float* red) {
    v = sum64(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    float s = 0.0f;
#pragma unroll
    for (int w = 0; w < WAVES; ++w) s += red[w];
    return s;
}

enum { GEMV_STORE = 0, GEMV_RELU2 = 1, GEMV_SIDE = 2, GEMV_ARGMAX = 3 };

// y = epilogue(W . prologue(x)).  Vectors are fp32, zero-padded to a multiple of 64 values.
// Prologue: x' = x + RMS(h) * hw + add0 + add1 (each part optional; x' stored to xout by one workgroup), then RMS(x') * gamma if
// gamma is given (stored to xn_out by one workgroup).
struct DenseGemv {
    const uint16_t* W = nullptr;
    int64_t ld = 0;
    int N = 0, K = 0;
    const float* x = nullptr;
    const float *h = nullptr, *hw = nullptr, *add0 = nullptr, *add1 = nullptr;
    float* xout = nullptr;
    const float* gamma = nullptr;
    float* xn_out = nullptr;
    float eps = 0.0f;
    int epilogue = GEMV_STORE;
    float* y = nullptr;
    const uint16_t* side = nullptr;  // GEMV_SIDE: row *d_token of the table, from column side_off
    int64_t side_ld = 0;
    int side_off = 0;
    const int* d_token = nullptr;
    float* part_val = nullptr;       // GEMV_ARGMAX: one (value, index) per workgroup
    int* part_idx = nullptr;
};
int dense_gemv_workgroups(const DenseGemv& g);
int dense_gemv(const DenseGemv& g, hipStream_t s);
void dense_gemv_init();

// One decode step of a latent mixer around its attention.
struct LatentStep {
    const float* proj;        // [heads * (dim + rot_dim)] q, then kv_rank latent values and rot_dim key values
    const float* c_norm;      // [kv_rank]
    const float* rope;        // [max_seq][rot.dims / 2][2]
    const uint16_t* expand;   // W_uk rows, then W_uv rows (per head padded to 8 rows)
    int64_t ld;
    int heads, dim, rot_dim, rot_dims, kv_rank, vdim;
    float eps;
    const int64_t* d_past;
    void* q;                  // [heads][up8(kv_rank) + up8(rot_dim)]: fp32, or two bfloat16 planes of that (tiled attention)
    int q_planes;
    void* cache;              // [max_seq][up8(kv_rank) + up8(rot_dim)]
    int fp32;
};
int latent_absorb(const LatentStep& a, hipStream_t s);
// out[h * up8(vdim) + v] = W_uv[h] . merged latent of head h; pM / pL NULL: pO is the finished latent [heads][o_row]
int latent_out(const LatentStep& a, const float* pO, const float* pM, const float* pL, int splits, int o_row, float* out,
               hipStream_t s);

// C = epilogue(A . W^T): GEMM_F32 fp32 C; otherwise element type of the rows (bfloat16, or fp32 when a_fp32)
enum { GEMM_F32 = 0, GEMM_ELEM = 1, GEMM_RELU2 = 2 };
struct DenseGemm {
    const void* A = nullptr;
    int a_fp32 = 0;
    int64_t lda = 0;
    const uint16_t* W = nullptr;
    int64_t ldw = 0;
    int M = 0, N = 0, K = 0;
    int epilogue = GEMM_F32;
    void* C = nullptr;
    int64_t ldc = 0;
    // K split over workgroups where the output has too few tiles (GEMM_F32 only): split z leaves its partial sums at
    // C + z * slab; slab_room floats are available for all of them
    int64_t slab = 0, slab_room = 0;
    int splits = 1;  // set by dense_gemm
};
int dense_gemm(DenseGemm g, hipStream_t s, int* splits = nullptr);

// Attention of one decode token, position *d_past.  bfloat16 caches with tile classes the matrix-core kernel has: splits
// partial results (decode_attention_splits); otherwise one finished result.
struct DecodeAttention {
    ptm_attention_args a;      // rows 1; Q (unless raw is given): two bfloat16 planes [2][heads][dim1 + dim2] that add up to q
    const int64_t* d_past;
    int max_seq;
    // attention mixer: un-normed projections, finished in the prologue, and the rows appended to the caches
    const float* raw = nullptr;  // [q | k | v]
    const float *q_norm = nullptr, *k_norm = nullptr, *rope = nullptr;
    int dim = 0, vdim_true = 0, rot_dims = 0;
    float eps = 0.0f;
    void *k_cache = nullptr, *v_cache = nullptr;
    float *pO = nullptr, *pM = nullptr, *pL = nullptr;  // [splits][heads][vdim], [splits][heads] twice
};
bool decode_attention_tiled(const ptm_attention_args& a);
int decode_attention_splits(const ptm_attention_args& a, int max_seq);
int decode_attention(const DecodeAttention& a, hipStream_t s);
int decode_attention_merge(const float* pO, const float* pM, const float* pL, int splits, int heads, int vdim, float* out,
                           hipStream_t s);
int attention_rows(const ptm_attention_args& a, const int64_t* d_past, bool q_fp32_out_fp32, hipStream_t s);

int argmax_finish(const float* part_val, const int* part_idx, int n, int64_t* out_index, const ArgmaxAdvance adv, hipStream_t s);

}  // namespace ptm
