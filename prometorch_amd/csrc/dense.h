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

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }

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

enum { GEMV_STORE = 0, GEMV_RELU2 = 1, GEMV_SIDE = 2, GEMV_ARGMAX = 3, GEMV_SWIGLU = 4 };
constexpr int GEMV_SECTIONS = 8;

// y = epilogue(W . prologue(x)).  Vectors are fp32, zero-padded to a multiple of 64 values.
// Prologue: x' = x + RMS(h) * hw + add0 + add1 (each part optional; x' stored to xout by one workgroup), then RMS(x') * gamma if
// gamma is given (stored to xn_out by one workgroup).
// With streams > 0, x is that many vectors x_stride floats apart: x' = sum_s blend[s] x_s + blend[streams] h, and with h the first
// workgroups store the new streams sum_s store[t][s] x_s + store[t][streams] h to xout (K-padded rows); layer norm if beta is
// given; then the token shift: rows of section i take x' + (x'_before - x') * mu[i], x'_before from the ring slot of the previous position.
// With tail_n > 0 (no other prologue), values tail0 .. of x are RMS-normed in tail_parts equal parts, times tail_norm * tail_scale.
// GEMV_SWIGLU: W holds N gate rows, then N up rows; y = silu(gate) * up.
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
    int streams = 0;
    int64_t x_stride = 0;
    const float *blend = nullptr, *store = nullptr, *beta = nullptr;
    const float* mu = nullptr;       // [sections][padded K]
    float* shift = nullptr;          // [2][padded K], by position parity
    const int64_t* d_past = nullptr;
    int sections = 0;
    int section_row[GEMV_SECTIONS + 1] = {};  // first rows; the last entry is N
    int section_wg[GEMV_SECTIONS + 1] = {};   // first workgroups, set by dense_gemv
    int tail0 = 0, tail_n = 0, tail_parts = 0;
    const float* tail_norm = nullptr;
    float tail_scale = 1.0f;
    float out_scale = 1.0f;          // factor of every stored y
};
int dense_gemv_workgroups(const DenseGemv& g);
int dense_gemv(DenseGemv g, hipStream_t s);
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

// C = epilogue(A . W^T): GEMM_F32 fp32 C; otherwise element type of the rows (bfloat16, or fp32 when a_fp32).
// GEMM_SWIGLU: W holds N / 2 gate rows, then N / 2 up rows; C [M][N / 2] = silu(gate) * up.
// GEMM_DECAY: fp32 C = exp(-exp(product + bias)).
enum { GEMM_F32 = 0, GEMM_ELEM = 1, GEMM_RELU2 = 2, GEMM_SWIGLU = 3, GEMM_DECAY = 4 };
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
    int splits = 1, tile_cols = 0;  // set by dense_gemm
    // rows n of W take A + n / section_n * section_a (section_n a multiple of 128; 0: one section)
    int section_n = 0;
    int64_t section_a = 0;
    const float* bias = nullptr;  // [N], GEMM_DECAY
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
    int head_norm = 0, values_are_keys = 0;  // q and k normed per head; v = the un-normed k
    void *k_cache = nullptr, *v_cache = nullptr;
    float *pO = nullptr, *pM = nullptr, *pL = nullptr;  // [splits][heads][vdim], [splits][heads] twice
};
bool decode_attention_tiled(const ptm_attention_args& a);
int decode_attention_splits(const ptm_attention_args& a, int max_seq);
int decode_attention(const DecodeAttention& a, hipStream_t s);
// a: heads, vdim, and the sink, gate and scale of the finished values
int decode_attention_merge(const float* pO, const float* pM, const float* pL, int splits, const ptm_attention_args& a, float* out,
                           hipStream_t s);
int attention_rows(const ptm_attention_args& a, const int64_t* d_past, bool q_fp32_out_fp32, hipStream_t s);

// ---- recurrent mixers (recurrent.hip) ----------------------------------------------------------
bool recurrent_supported(int keys);
int64_t recurrent_state_floats(int heads, int keys, int columns);

struct WkvStep {
    const float* proj;        // [r | k | v | g | low-rank]
    const uint16_t* w2;       // [heads * dim][w2_ld]
    int64_t w2_ld;
    int heads, dim, rank;
    const float *w0, *u, *norm;
    float eps;
    const int64_t* d_past;
    float* state;
    float* out;               // [heads * dim]
};
int wkv_step(const WkvStep& a, hipStream_t s);

struct WkvRows {
    const float* proj;        // [M][ld]: r, k, v, g and the decays w, `section` floats apart
    int64_t ld, section;
    int M, heads, dim;
    const float *u, *norm;
    float eps;
    int64_t pos0;
    float* state;
    float* o;                 // [scan_slabs(dim)][M][o_ld], o_slab floats apart
    int64_t o_ld, o_slab;
    int groups;               // set by wkv_rows
    void* out;                // [M][out_ld]
    int64_t out_ld;
    const float* h_last;      // the mixer's last input row, kept for the next token's shift
    float* shift;
    int wp;
};
int wkv_rows(WkvRows a, bool fp32, hipStream_t s);
int64_t scan_slabs(int keys);  // partial sums that a scan leaves per row
int token_shift_rows(const float* h, const float* shift, const float* mu, int n, int rows, int64_t pos0, int wp, bool fp32, void* out, hipStream_t s);
int tanh_rows(const float* g, int slabs, int64_t slab, int rows, int n, bool fp32, void* out, hipStream_t s);

struct SsmShape {
    int heads, vdim, state, groups, taps, norm_groups;
    const float *conv, *conv_b, *dt_bias, *neg_a, *D, *norm;  // neg_a: -exp(A_log)
    float scale;
};
struct SsmStep {
    SsmShape m;
    const float* proj;        // [z | x | B | C | dt]
    const int64_t* d_past;
    float *ring, *state;      // [taps][channels]; state
    float* out;               // [heads * vdim], before its norm
};
int ssm_step(const SsmStep& a, hipStream_t s);
struct SsmRows {
    SsmShape m;
    const float* proj;        // [M][ld]
    int64_t ld;
    int M;
    int64_t pos0;
    float eps;
    float *ring, *state;
    float* conv;              // [M][x | B | C]
    float* decay;             // [M][2][heads]
    float* y;                 // [scan_slabs(state)][M][heads * vdim], y_slab floats apart
    int64_t y_slab;
    int key_groups;           // set by ssm_rows
    void* out;                // [M][out_ld]
    int64_t out_ld;
};
int ssm_rows(SsmRows a, bool fp32, hipStream_t s);

int argmax_finish(const float* part_val, const int* part_idx, int n, int64_t* out_index, const ArgmaxAdvance adv, hipStream_t s);

}  // namespace ptm
