// Prompt products over bfloat16 weights: C[M][N] = A[M][K] . W[N][K]^T on the matrix cores.
//
// dense_gemm_kernel (bfloat16 rows): 4 waves, BM x BN output tile, 64 values of K per step.  Tiles go global -> registers ->
// LDS; two register sets and two LDS buffers, so a step has one barrier and the loads of the next two steps are in flight
// while its MFMAs run.
// LDS rows are 128 bytes, the eight 16-byte pieces of row r stored at piece ^ (r % 8): the fragment reads (32 rows, one
// piece) and the writes touch every bank evenly.  The product is formed transposed (W rows as the A operand), so that a lane
// holds four consecutive columns of one output row.
// dense_gemm_f32_kernel (fp32 rows): the same product in fp32 on v_mfma_f32_32x32x2_f32, 64 x 64 tiles.
#include "dense.h"

namespace ptm {

typedef __bf16 gm_b8 __attribute__((ext_vector_type(8)));
typedef float gm_f16 __attribute__((ext_vector_type(16)));

// workgroups are dealt to the 8 XCDs in turn: give each XCD a contiguous run of tiles (rows fastest, so a run shares columns of W)
__device__ __forceinline__ void tile_of(int wg, int tiles_m, int tiles_n, int& tm, int& tn) {
    const int total = tiles_m * tiles_n, per = total / 8, rem = total % 8, xcd = wg % 8, i = wg / 8;
    const int id = xcd * per + min(xcd, rem) + i;
    tm = id % tiles_m;
    tn = id / tiles_m;
}

__device__ __forceinline__ float relu2(float v) { return v > 0.0f ? v * v : 0.0f; }

// row of W behind column n of the product.  GEMM_SWIGLU: each 32 columns are 16 gate rows and the 16 up rows of the same values,
// which one lane's accumulators hold together.
__device__ __forceinline__ int weight_row(const DenseGemm& g, int n) {
    if (g.epilogue != GEMM_SWIGLU) return min(n, g.N - 1);
    const int ff = g.N / 2, v = min((n >> 5) * 16 + (n & 15), ff - 1);
    return (n & 16) ? ff + v : v;
}

// four consecutive columns n .. n + 3 of row m
template <bool F32>
__device__ __forceinline__ void store4(const DenseGemm& g, int split, int m, int n, float v0, float v1, float v2, float v3) {
    if (g.epilogue == GEMM_RELU2) {
        v0 = relu2(v0);
        v1 = relu2(v1);
        v2 = relu2(v2);
        v3 = relu2(v3);
    }
    if (g.epilogue == GEMM_DECAY) {
        auto decay = [&](float v, int k) { return k < g.N ? expf(-expf(v + g.bias[k])) : 0.0f; };
        v0 = decay(v0, n);
        v1 = decay(v1, n + 1);
        v2 = decay(v2, n + 2);
        v3 = decay(v3, n + 3);
    }
    const int64_t at = (int64_t)m * g.ldc + n + split * g.slab;
    if (F32 || g.epilogue == GEMM_F32 || g.epilogue == GEMM_DECAY) {
        float* c = static_cast<float*>(g.C) + at;
        if (n + 3 < g.N && (g.ldc & 3) == 0) {
            *reinterpret_cast<float4*>(c) = make_float4(v0, v1, v2, v3);
        } else {
            c[0] = v0;
            if (n + 1 < g.N) c[1] = v1;
            if (n + 2 < g.N) c[2] = v2;
            if (n + 3 < g.N) c[3] = v3;
        }
    } else {
        uint16_t* c = static_cast<uint16_t*>(g.C) + at;
        if (n + 3 < g.N && (g.ldc & 3) == 0) {
            *reinterpret_cast<uint2*>(c) = make_uint2((uint32_t)f_bf16(v0) | ((uint32_t)f_bf16(v1) << 16), (uint32_t)f_bf16(v2) | ((uint32_t)f_bf16(v3) << 16));
        } else {
            c[0] = f_bf16(v0);
            if (n + 1 < g.N) c[1] = f_bf16(v1);
            if (n + 2 < g.N) c[2] = f_bf16(v2);
            if (n + 3 < g.N) c[3] = f_bf16(v3);
        }
    }
}

// 32 columns of GEMM_SWIGLU: accumulators 0..7 are gates, 8..15 the ups of the same values
template <bool F32>
__device__ __forceinline__ void store_glu(const DenseGemm& g, int m, int n, int kh, const gm_f16& acc) {
    DenseGemm o = g;
    o.epilogue = GEMM_ELEM;
    o.N = g.N / 2;
#pragma unroll
    for (int q = 0; q < 2; ++q) {
        const int v = n / 2 + 8 * q + 4 * kh;
        if (v < o.N)
            store4<F32>(o, 0, m, v, silu_f(acc[4 * q]) * acc[8 + 4 * q], silu_f(acc[4 * q + 1]) * acc[9 + 4 * q],
                        silu_f(acc[4 * q + 2]) * acc[10 + 4 * q], silu_f(acc[4 * q + 3]) * acc[11 + 4 * q]);
    }
}

template <int BM, int BN, int WM, int WN>
__global__ __launch_bounds__(256, 2) void dense_gemm_kernel(const DenseGemm g) {
    static_assert((BM / WM) * (BN / WN) == 4, "four waves");
    constexpr int TM = WM / 32, TN = WN / 32, PA = BM / 32, PB = BN / 32;  // pieces of 16 bytes a thread stages
    __shared__ __align__(16) uint8_t s_a[2][BM * 128];
    __shared__ __align__(16) uint8_t s_b[2][BN * 128];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int j = lane & 31, kh = lane >> 5;
    int tm, tn;
    const int tiles_m = (g.M + BM - 1) / BM, tiles_n = (g.tile_cols + BN - 1) / BN, split = blockIdx.x / (tiles_m * tiles_n);
    tile_of(blockIdx.x - split * tiles_m * tiles_n, tiles_m, tiles_n, tm, tn);
    const int m0 = tm * BM, n0 = tn * BN;
    const int wm = (wave % (BM / WM)) * WM, wn = (wave / (BM / WM)) * WN;
    const int all = (g.K + 63) / 64, steps = all * (split + 1) / g.splits, first = all * split / g.splits;
    const uint16_t* A = static_cast<const uint16_t*>(g.A);
    if (g.section_n > 0) A += n0 / g.section_n * g.section_a;
    const int pr = tid >> 3, pp = tid & 7;  // row and piece of this thread's first staged piece; the others 32 rows on
    const u32x4* pa[PA];
    const u32x4* pb[PB];
    uint32_t la[PA], lb[PB];
#pragma unroll
    for (int i = 0; i < PA; ++i) {
        const int r = pr + 32 * i;
        pa[i] = reinterpret_cast<const u32x4*>(A + (int64_t)min(m0 + r, g.M - 1) * g.lda) + pp;
        la[i] = r * 128 + ((pp ^ (r & 7)) << 4);
    }
#pragma unroll
    for (int i = 0; i < PB; ++i) {
        const int r = pr + 32 * i;
        pb[i] = reinterpret_cast<const u32x4*>(g.W + (int64_t)weight_row(g, n0 + r) * g.ldw) + pp;
        lb[i] = r * 128 + ((pp ^ (r & 7)) << 4);
    }
    u32x4 ra0[PA], rb0[PB], ra1[PA], rb1[PB];
    auto fetch = [&](int st, u32x4 (&ra)[PA], u32x4 (&rb)[PB]) {
        st = st < steps ? st : steps - 1;
#pragma unroll
        for (int i = 0; i < PA; ++i) ra[i] = pa[i][st * 8];
#pragma unroll
        for (int i = 0; i < PB; ++i) rb[i] = pb[i][st * 8];
    };
    auto stage = [&](int buf, const u32x4 (&ra)[PA], const u32x4 (&rb)[PB]) {
#pragma unroll
        for (int i = 0; i < PA; ++i) *reinterpret_cast<u32x4*>(&s_a[buf][la[i]]) = ra[i];
#pragma unroll
        for (int i = 0; i < PB; ++i) *reinterpret_cast<u32x4*>(&s_b[buf][lb[i]]) = rb[i];
    };
    gm_f16 acc[TM][TN];
#pragma unroll
    for (int a = 0; a < TM; ++a)
#pragma unroll
        for (int b = 0; b < TN; ++b)
#pragma unroll
            for (int r = 0; r < 16; ++r) acc[a][b][r] = 0.0f;
    auto multiply = [&](int buf) {
#pragma unroll
        for (int ks = 0; ks < 4; ++ks) {
            const int pc = ((2 * ks + kh) ^ (j & 7)) << 4;
            gm_b8 fa[TM], fb[TN];
#pragma unroll
            for (int a = 0; a < TM; ++a) fa[a] = *reinterpret_cast<const gm_b8*>(&s_a[buf][(wm + 32 * a + j) * 128 + pc]);
#pragma unroll
            for (int b = 0; b < TN; ++b) fb[b] = *reinterpret_cast<const gm_b8*>(&s_b[buf][(wn + 32 * b + j) * 128 + pc]);
#pragma unroll
            for (int a = 0; a < TM; ++a)
#pragma unroll
                for (int b = 0; b < TN; ++b) acc[a][b] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fb[b], fa[a], acc[a][b], 0, 0, 0);
        }
    };
    fetch(first, ra0, rb0);
    fetch(first + 1, ra1, rb1);
    stage(0, ra0, rb0);
    __syncthreads();
    // two steps per trip; a step past the end repeats the last one's loads and is not multiplied
    for (int st = first; st < steps; st += 2) {
        fetch(st + 2, ra0, rb0);
        multiply(0);
        stage(1, ra1, rb1);
        __syncthreads();
        fetch(st + 3, ra1, rb1);
        if (st + 1 < steps) multiply(1);
        stage(0, ra0, rb0);
        __syncthreads();
    }
#pragma unroll
    for (int a = 0; a < TM; ++a) {
        const int m = m0 + wm + 32 * a + j;
        if (m >= g.M) continue;
#pragma unroll
        for (int b = 0; b < TN; ++b) {
            if (g.epilogue == GEMM_SWIGLU) {
                store_glu<false>(g, m, n0 + wn + 32 * b, kh, acc[a][b]);
                continue;
            }
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                const int n = n0 + wn + 32 * b + 8 * q + 4 * kh;
                if (n < g.N) store4<false>(g, split, m, n, acc[a][b][4 * q], acc[a][b][4 * q + 1], acc[a][b][4 * q + 2], acc[a][b][4 * q + 3]);
            }
        }
    }
}

__global__ __launch_bounds__(256) void dense_gemm_f32_kernel(const DenseGemm g) {
    constexpr int BK = 32, P = BK + 1;
    __shared__ float s_a[64 * P], s_b[64 * P];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, j = lane & 31, kh = lane >> 5;
    int tm, tn;
    tile_of(blockIdx.x, (g.M + 63) / 64, (g.tile_cols + 63) / 64, tm, tn);
    const int m0 = tm * 64, n0 = tn * 64, wm = (wave & 1) * 32, wn = (wave >> 1) * 32;
    const float* A = static_cast<const float*>(g.A);
    if (g.section_n > 0) A += n0 / g.section_n * g.section_a;
    gm_f16 acc;
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[r] = 0.0f;
    const int r0 = tid >> 2, c0 = (tid & 3) * 8;
    const float* pa = A + (int64_t)min(m0 + r0, g.M - 1) * g.lda + c0;
    const uint16_t* pb = g.W + (int64_t)weight_row(g, n0 + r0) * g.ldw + c0;
    const int steps = (g.K + BK - 1) / BK;
    for (int st = 0; st < steps; ++st) {
        const float4 a0 = *reinterpret_cast<const float4*>(pa + st * BK), a1 = *reinterpret_cast<const float4*>(pa + st * BK + 4);
        const uint4 w = *reinterpret_cast<const uint4*>(pb + st * BK);
        __syncthreads();
        float* d = s_a + r0 * P + c0;
        d[0] = a0.x; d[1] = a0.y; d[2] = a0.z; d[3] = a0.w; d[4] = a1.x; d[5] = a1.y; d[6] = a1.z; d[7] = a1.w;
        d = s_b + r0 * P + c0;
        d[0] = bf16_lo(w.x); d[1] = bf16_hi(w.x); d[2] = bf16_lo(w.y); d[3] = bf16_hi(w.y);
        d[4] = bf16_lo(w.z); d[5] = bf16_hi(w.z); d[6] = bf16_lo(w.w); d[7] = bf16_hi(w.w);
        __syncthreads();
#pragma unroll
        for (int k = 0; k < BK; k += 2)
            acc = __builtin_amdgcn_mfma_f32_32x32x2f32(s_b[(wn + j) * P + k + kh], s_a[(wm + j) * P + k + kh], acc, 0, 0, 0);
    }
    const int m = m0 + wm + j;
    if (m >= g.M) return;
    if (g.epilogue == GEMM_SWIGLU) return store_glu<true>(g, m, n0 + wn, kh, acc);
#pragma unroll
    for (int q = 0; q < 4; ++q) {
        const int n = n0 + wn + 8 * q + 4 * kh;
        if (n < g.N) store4<true>(g, 0, m, n, acc[4 * q], acc[4 * q + 1], acc[4 * q + 2], acc[4 * q + 3]);
    }
}

int dense_gemm(DenseGemm g, hipStream_t s, int* splits) {
    if (!g.A || !g.W || !g.C) return PTM_E_NULL;
    const int kp = up64(g.K);
    const bool glu = g.epilogue == GEMM_SWIGLU;
    if (g.M <= 0 || g.N <= 0 || g.K <= 0 || g.lda <= 0 || g.ldw < kp || g.ldc < (glu ? g.N / 2 : g.N)) return PTM_E_SHAPE;
    if ((glu && (g.N & 1)) || g.section_n < 0 || (g.section_n & 127) || (g.section_a & 7)) return PTM_E_SHAPE;
    if (g.epilogue != GEMM_F32 && splits) return PTM_E_SHAPE;  // partial sums have no epilogue
    if (g.epilogue == GEMM_DECAY && !g.bias) return PTM_E_NULL;
    if (!aligned16(g.A) || !aligned16(g.W) || !aligned16(g.C) || (g.lda & 7) || (g.ldw & 7)) return PTM_E_ALIGN;
    const int cols = glu ? (g.N / 2 + 15) / 16 * 32 : g.N;  // gates and ups in whole blocks of 16
    g.tile_cols = cols;
    auto tiles = [&](int bm, int bn) { return ((int64_t)g.M + bm - 1) / bm * ((cols + bn - 1) / bn); };
    if (tiles(32, 64) * 16 > 0x7fffffff) return PTM_E_UNSUPPORTED;
    // splits that bring `t` tiles to about `target` workgroups, each with at least four steps of K
    auto split = [&](int64_t t, int64_t target) {
        g.splits = 1;
        if (!splits || g.slab <= 0) return;
        int64_t n = (target + t / 2) / t;
        if (n > kp / 256) n = kp / 256;
        if (n > 16) n = 16;
        while (n > 1 && n * g.slab > g.slab_room) --n;
        g.splits = n > 1 ? (int)n : 1;
    };
    if (g.a_fp32) {
        g.splits = 1;
        hipLaunchKernelGGL(dense_gemm_f32_kernel, dim3((unsigned)tiles(64, 64)), dim3(256), 0, s, g);
    } else if (g.M <= 32) {
        split(tiles(32, 128), 512);
        hipLaunchKernelGGL((dense_gemm_kernel<32, 128, 32, 32>), dim3((unsigned)(tiles(32, 128) * g.splits)), dim3(256), 0, s, g);
    } else if (g.M <= 64) {
        split(tiles(64, 64), 512);
        hipLaunchKernelGGL((dense_gemm_kernel<64, 64, 32, 32>), dim3((unsigned)(tiles(64, 64) * g.splits)), dim3(256), 0, s, g);
    } else {
        const int64_t t = tiles(128, 128);
        if (t < 192) split(t, 384);
        if (t * g.splits >= 128)
            hipLaunchKernelGGL((dense_gemm_kernel<128, 128, 64, 64>), dim3((unsigned)(t * g.splits)), dim3(256), 0, s, g);
        else
            hipLaunchKernelGGL((dense_gemm_kernel<64, 64, 32, 32>), dim3((unsigned)(tiles(64, 64) * g.splits)), dim3(256), 0, s, g);
    }
    if (splits) *splits = g.splits;
    return launch_status();
}

}  // namespace ptm

extern "C" int ptm_dense_gemm(const void* A, int a_fp32, int64_t lda, const void* W, int64_t ldw, float* C, int64_t ldc, int M,
                              int N, int K, ptm_stream_t stream) {
    if (M <= 0 || N <= 0 || K <= 0 || lda < ptm::up64(K)) return PTM_E_SHAPE;
    ptm::DenseGemm g;
    g.A = A;
    g.a_fp32 = a_fp32;
    g.lda = lda;
    g.W = static_cast<const uint16_t*>(W);
    g.ldw = ldw;
    g.M = M;
    g.N = N;
    g.K = K;
    g.C = C;
    g.ldc = ldc;
    return ptm::dense_gemm(g, ptm::as_stream(stream));
}
