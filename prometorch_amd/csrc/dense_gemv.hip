// Decode products over bfloat16 weights: y = W . x with fp32 activations, and the two products a latent-attention step
// makes around its attention.
//
// dense_gemv_kernel: 8 waves per workgroup; LPR lanes share a row (64; fewer for short rows), each taking 8 values (16 bytes)
// per chunk, R rows x U chunks in flight per lane, the next batch requested before the current one is consumed.  The
// activation vector lies in LDS as fp32, the two halves of every 8 values in separate planes so that a wave's 16-byte reads
// are consecutive.  The first weight batch is requested before the prologue, which forms the vector: deferred post-norm and
// residual add, loop inputs, RMSNorm - recomputed by every workgroup, as the quantised kernels do.
#include "dense.h"

namespace ptm {

constexpr int DG_WAVES = 8, DG_THREADS = 64 * DG_WAVES;

__device__ __forceinline__ float4 ld4(const float* p, int i) { return reinterpret_cast<const float4*>(p)[i]; }
__device__ __forceinline__ float sq4(float4 v, float s) {
    s = fmaf(v.x, v.x, s);
    s = fmaf(v.y, v.y, s);
    s = fmaf(v.z, v.z, s);
    return fmaf(v.w, v.w, s);
}
__device__ __forceinline__ float4 add4(float4 a, float4 b) { return make_float4(a.x + b.x, a.y + b.y, a.z + b.z, a.w + b.w); }

template <int LPR, int R, int U, bool PRO>
__global__ __launch_bounds__(DG_THREADS, 4) void dense_gemv_kernel(const DenseGemv a) {
    extern __shared__ __align__(16) float4 s_x[];  // [2][Kp / 8]
    __shared__ float red[DG_WAVES];
    __shared__ int redi[DG_WAVES];
    constexpr int RPP = 64 / LPR, RW = RPP * R;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int li = lane % LPR, lr = lane / LPR;
    const int Kp = (a.K + 63) & ~63, n4 = Kp / 4, n8 = Kp / 8;
    const int groups = (a.N + RW - 1) / RW, stride = gridDim.x * DG_WAVES;
    const int nb = (n8 + LPR * U - 1) / (LPR * U);
    const uint32_t bytes = (uint32_t)((int64_t)a.N * a.ld * 2);
    const __amdgpu_buffer_rsrc_t rs = make_rsrc(a.W, (int)bytes);
    auto load = [&](int g, int b, u32x4* w) {
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const int row = min(g * RW + r * RPP + lr, a.N - 1);
            const uint32_t base = (uint32_t)row * (uint32_t)(a.ld * 2);
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int kk = (b * U + u) * LPR + li;
                w[r * U + u] = __builtin_amdgcn_raw_buffer_load_b128(rs, kk < n8 ? base + (uint32_t)kk * 16u : bytes, 0, 0);
            }
        }
    };
    auto put = [&](int i, float4 v) { s_x[(i & 1) * n8 + (i >> 1)] = v; };

    u32x4 cur[R * U], nxt[R * U];
    int g = blockIdx.x * DG_WAVES + wave, b = 0;
    if constexpr (!PRO) {
        for (int i = tid; i < n4; i += DG_THREADS) put(i, ld4(a.x, i));
        load(min(g, groups - 1), 0, cur);
        __syncthreads();
    } else {
        const bool first = blockIdx.x == 0;
        if (n4 <= 2 * DG_THREADS) {  // the vector stays in registers between the passes
            const float4 z = make_float4(0.f, 0.f, 0.f, 0.f);
            float4 xv[2] = {z, z}, hv[2] = {z, z}, wv[2] = {z, z}, gv[2] = {z, z};
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                const int i = tid + u * DG_THREADS;
                if (i < n4) {
                    if (a.h) { hv[u] = ld4(a.h, i); wv[u] = ld4(a.hw, i); }
                    xv[u] = ld4(a.x, i);
                    if (a.add0) xv[u] = add4(xv[u], ld4(a.add0, i));
                    if (a.add1) xv[u] = add4(xv[u], ld4(a.add1, i));
                    if (a.gamma) gv[u] = ld4(a.gamma, i);
                }
            }
            issue_order_fence();
            load(min(g, groups - 1), 0, cur);
            if (a.h) {
                const float r = 1.0f / sqrtf(block_sum<DG_WAVES>(sq4(hv[1], sq4(hv[0], 0.f)), red) / (float)a.K + a.eps);
#pragma unroll
                for (int u = 0; u < 2; ++u)
                    xv[u] = add4(xv[u], make_float4(hv[u].x * r * wv[u].x, hv[u].y * r * wv[u].y, hv[u].z * r * wv[u].z, hv[u].w * r * wv[u].w));
            }
            float r = 1.0f;
            if (a.gamma) r = 1.0f / sqrtf(block_sum<DG_WAVES>(sq4(xv[1], sq4(xv[0], 0.f)), red) / (float)a.K + a.eps);
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                const int i = tid + u * DG_THREADS;
                if (i < n4) {
                    if (first && a.xout) reinterpret_cast<float4*>(a.xout)[i] = xv[u];
                    float4 v = xv[u];
                    if (a.gamma) v = make_float4(v.x * r * gv[u].x, v.y * r * gv[u].y, v.z * r * gv[u].z, v.w * r * gv[u].w);
                    if (first && a.xn_out) reinterpret_cast<float4*>(a.xn_out)[i] = v;
                    put(i, v);
                }
            }
        } else {  // long vectors: kept in LDS between the passes
            load(min(g, groups - 1), 0, cur);
            float rh = 0.0f;
            if (a.h) {
                float ss = 0.0f;
                for (int i = tid; i < n4; i += DG_THREADS) ss = sq4(ld4(a.h, i), ss);
                rh = 1.0f / sqrtf(block_sum<DG_WAVES>(ss, red) / (float)a.K + a.eps);
            }
            float ss = 0.0f;
            for (int i = tid; i < n4; i += DG_THREADS) {
                float4 v = ld4(a.x, i);
                if (a.add0) v = add4(v, ld4(a.add0, i));
                if (a.add1) v = add4(v, ld4(a.add1, i));
                if (a.h) {
                    const float4 h = ld4(a.h, i), w = ld4(a.hw, i);
                    v = add4(v, make_float4(h.x * rh * w.x, h.y * rh * w.y, h.z * rh * w.z, h.w * rh * w.w));
                }
                if (first && a.xout) reinterpret_cast<float4*>(a.xout)[i] = v;
                ss = sq4(v, ss);
                put(i, v);
            }
            if (a.gamma) {
                const float r = 1.0f / sqrtf(block_sum<DG_WAVES>(ss, red) / (float)a.K + a.eps);
                for (int i = tid; i < n4; i += DG_THREADS) {  // a thread rescales the slots it wrote itself
                    const float4 gm = ld4(a.gamma, i);
                    float4 v = s_x[(i & 1) * n8 + (i >> 1)];
                    v = make_float4(v.x * r * gm.x, v.y * r * gm.y, v.z * r * gm.z, v.w * r * gm.w);
                    if (first && a.xn_out) reinterpret_cast<float4*>(a.xn_out)[i] = v;
                    put(i, v);
                }
            }
        }
        __syncthreads();
    }

    const int64_t side_row = a.epilogue == GEMV_SIDE ? (int64_t)*a.d_token * a.side_ld + a.side_off : 0;
    float best = -INFINITY;
    int best_i = 0x7fffffff;
    float acc[R];
#pragma unroll
    for (int r = 0; r < R; ++r) acc[r] = 0.0f;
    while (g < groups) {
        const bool last = b + 1 == nb;
        const int ng = last ? g + stride : g, nbb = last ? 0 : b + 1;
        if (ng < groups) load(ng, nbb, nxt);
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int kk = (b * U + u) * LPR + li, kc = min(kk, n8 - 1);  // a chunk past the end holds zero weights
            const float4 x0 = s_x[kc], x1 = s_x[n8 + kc];
#pragma unroll
            for (int r = 0; r < R; ++r) {
                const u32x4 w = cur[r * U + u];
                float t = acc[r];
                t = fmaf(bf16_lo(w.x), x0.x, t);
                t = fmaf(bf16_hi(w.x), x0.y, t);
                t = fmaf(bf16_lo(w.y), x0.z, t);
                t = fmaf(bf16_hi(w.y), x0.w, t);
                t = fmaf(bf16_lo(w.z), x1.x, t);
                t = fmaf(bf16_hi(w.z), x1.y, t);
                t = fmaf(bf16_lo(w.w), x1.z, t);
                t = fmaf(bf16_hi(w.w), x1.w, t);
                acc[r] = t;
            }
        }
        if (last) {
#pragma unroll
            for (int r = 0; r < R; ++r) {
                float v = LPR == 64 ? sum64(acc[r]) : sum_lanes<LPR == 64 ? 32 : LPR>(acc[r]);
                acc[r] = 0.0f;
                const int row = g * RW + r * RPP + lr;
                if (li == 0 && row < a.N) {
                    if (a.epilogue == GEMV_RELU2) v = v > 0.0f ? v * v : 0.0f;
                    else if (a.epilogue == GEMV_SIDE) v = gelu_tanh(v) * bf16_f(a.side[side_row + row]);
                    else if (a.epilogue == GEMV_ARGMAX && (v > best || (v == best && row < best_i))) { best = v; best_i = row; }
                    a.y[row] = v;
                }
            }
        }
#pragma unroll
        for (int i = 0; i < R * U; ++i) cur[i] = nxt[i];
        g = ng;
        b = nbb;
    }
    if (a.epilogue == GEMV_ARGMAX) {
        for (int off = 1; off < 64; off <<= 1) {
            const float ov = __shfl_xor(best, off, 64);
            const int oi = __shfl_xor(best_i, off, 64);
            if (ov > best || (ov == best && oi < best_i)) { best = ov; best_i = oi; }
        }
        __syncthreads();
        if (lane == 0) { red[wave] = best; redi[wave] = best_i; }
        __syncthreads();
        if (tid == 0) {
            for (int w = 1; w < DG_WAVES; ++w)
                if (red[w] > best || (red[w] == best && redi[w] < best_i)) { best = red[w]; best_i = redi[w]; }
            a.part_val[blockIdx.x] = best;
            a.part_idx[blockIdx.x] = best_i;
        }
    }
}

namespace {
struct GemvShape { int kind, rows_per_wave; };
// rows shorter than a wave's 512 values share a wave; long rows take more chunks of one row, short ones more rows
GemvShape gemv_shape(const DenseGemv& g) {
    const int kp = up64(g.K), ch = (kp + 511) / 512;
    if (kp <= 64) return {0, 32};
    if (kp <= 256) return {1, 8};
    const bool few = g.N <= 2 * DG_WAVES * 256;  // two rows per wave would leave compute units without work
    if (ch <= 2) return few ? GemvShape{5, 1} : GemvShape{2, 4};
    if (ch <= 4 || (ch <= 7 && !few)) return few ? GemvShape{5, 1} : GemvShape{3, 2};
    return {4, 1};
}
}  // namespace

int dense_gemv_workgroups(const DenseGemv& g) {
    const int groups = (g.N + gemv_shape(g).rows_per_wave - 1) / gemv_shape(g).rows_per_wave;
    const int wgs = (groups + DG_WAVES - 1) / DG_WAVES;
    return wgs < 512 ? wgs : 512;
}

template <bool PRO>
static void gemv_attr() {
    const int lds = 150 * 1024;
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(dense_gemv_kernel<8, 4, 1, PRO>), hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(dense_gemv_kernel<32, 4, 1, PRO>), hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(dense_gemv_kernel<64, 4, 2, PRO>), hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(dense_gemv_kernel<64, 2, 4, PRO>), hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(dense_gemv_kernel<64, 1, 8, PRO>), hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(dense_gemv_kernel<64, 1, 4, PRO>), hipFuncAttributeMaxDynamicSharedMemorySize, lds);
}
// one-time kernel attributes, before anything can be captured
void dense_gemv_init() {
    gemv_attr<false>();
    gemv_attr<true>();
}

int dense_gemv(const DenseGemv& g, hipStream_t s) {
    if (!g.W || !g.x || !g.y) return PTM_E_NULL;
    if (g.N <= 0 || g.K <= 0 || g.ld < up64(g.K)) return PTM_E_SHAPE;
    if (up64(g.K) > 36864 || (int64_t)g.N * g.ld * 2 >= (int64_t)0xfffffff0u) return PTM_E_UNSUPPORTED;
    if (!aligned16(g.W) || !aligned16(g.x) || (g.ld & 7)) return PTM_E_ALIGN;
    const dim3 grid(dense_gemv_workgroups(g)), block(DG_THREADS);
    const size_t lds = (size_t)up64(g.K) * 4;
    const bool pro = g.h || g.add0 || g.add1 || g.gamma || g.xout || g.xn_out;
#define PTM_DG(LPR, R, U)                                                                            \
    if (pro) hipLaunchKernelGGL((dense_gemv_kernel<LPR, R, U, true>), grid, block, lds, s, g);       \
    else hipLaunchKernelGGL((dense_gemv_kernel<LPR, R, U, false>), grid, block, lds, s, g)
    switch (gemv_shape(g).kind) {
        case 0: PTM_DG(8, 4, 1); break;
        case 1: PTM_DG(32, 4, 1); break;
        case 2: PTM_DG(64, 4, 2); break;
        case 3: PTM_DG(64, 2, 4); break;
        case 4: PTM_DG(64, 1, 8); break;
        default: PTM_DG(64, 1, 4); break;
    }
#undef PTM_DG
    return launch_status();
}

// ---- latent attention ----------------------------------------------------------------------------
// grid heads * ceil(kv_rank / 128) + 1.  A workgroup (head, run of 128 latent dimensions): q[h][r] = sum_d q_unrotated[h][d]
// W_uk[h, d][r]; 16 lanes take 8 consecutive r each, the 16 lane groups stride over d, summed through LDS.  The first
// run's workgroup also rotates the head's rotated part.  The last workgroup norms the token's latent, rotates its key part and
// appends both to the cache.
template <bool F32>
__global__ __launch_bounds__(256) void latent_absorb_kernel(const LatentStep a) {
    __shared__ float s_q[1024];
    __shared__ float s_sum[16][128];
    __shared__ float red[4];
    const int tid = threadIdx.x;
    const int rank8 = (a.kv_rank + 7) & ~7, rot8 = (a.rot_dim + 7) & ~7, row = rank8 + rot8, qd = a.dim + a.rot_dim;
    const int runs = (a.kv_rank + 127) / 128, half = a.rot_dims / 2;
    const int64_t past = *a.d_past;
    const float* cs = a.rope + past * a.rot_dims;
    if ((int)blockIdx.x == a.heads * runs) {
        const float* src = a.proj + (int64_t)a.heads * qd;
        float ss = 0.0f;
        for (int i = tid; i < a.kv_rank; i += 256) ss = fmaf(src[i], src[i], ss);
        const float r = 1.0f / sqrtf(block_sum<4>(ss, red) / (float)a.kv_rank + a.eps);
        const int64_t base = past * row;
        for (int i = tid; i < rank8; i += 256) put_elem<F32>(a.cache, base + i, i < a.kv_rank ? src[i] * r * a.c_norm[i] : 0.0f);
        for (int i = tid; i < rot8; i += 256) {
            float v = 0.0f;
            if (i < a.rot_dim) {
                v = src[a.kv_rank + i];
                if (i < a.rot_dims) {
                    const float c = cs[2 * (i >> 1)], sn = cs[2 * (i >> 1) + 1], o = src[a.kv_rank + (i ^ 1)];
                    v = (i & 1) ? v * c + o * sn : v * c - o * sn;
                }
            }
            put_elem<F32>(a.cache, base + rank8 + i, v);
        }
        return;
    }
    const int h = blockIdx.x / runs, r0 = (blockIdx.x % runs) * 128;
    const int dim8 = (a.dim + 7) & ~7;
    const int lr = tid & 15, dg = tid >> 4, rr = r0 + lr * 8;
    const float* q = a.proj + (int64_t)h * qd;
    const uint16_t* w = a.expand + ((int64_t)h * dim8) * a.ld + (rr < a.kv_rank ? rr : 0);
    u32x4 wr[8];  // the first 128 rows, requested before q is staged
#pragma unroll
    for (int u = 0; u < 8; ++u) wr[u] = *reinterpret_cast<const u32x4*>(w + (int64_t)min(dg + 16 * u, a.dim - 1) * a.ld);
    for (int i = tid; i < a.dim; i += 256) s_q[i] = q[i];
    __syncthreads();
    float acc[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) acc[i] = 0.0f;
    auto add = [&](const u32x4& v, float x) {
        acc[0] = fmaf(bf16_lo(v.x), x, acc[0]);
        acc[1] = fmaf(bf16_hi(v.x), x, acc[1]);
        acc[2] = fmaf(bf16_lo(v.y), x, acc[2]);
        acc[3] = fmaf(bf16_hi(v.y), x, acc[3]);
        acc[4] = fmaf(bf16_lo(v.z), x, acc[4]);
        acc[5] = fmaf(bf16_hi(v.z), x, acc[5]);
        acc[6] = fmaf(bf16_lo(v.w), x, acc[6]);
        acc[7] = fmaf(bf16_hi(v.w), x, acc[7]);
    };
    if (rr < a.kv_rank) {
#pragma unroll
        for (int u = 0; u < 8; ++u) add(wr[u], dg + 16 * u < a.dim ? s_q[dg + 16 * u] : 0.0f);
#pragma unroll 4
        for (int d = dg + 128; d < a.dim; d += 16) add(*reinterpret_cast<const u32x4*>(w + (int64_t)d * a.ld), s_q[d]);
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) s_sum[dg][lr * 8 + i] = acc[i];
    __syncthreads();
    auto put_q = [&](int i, float v) {
        const int64_t at = (int64_t)h * row + i;
        if (a.q_planes) {
            const uint16_t hi = f_bf16(v);
            static_cast<uint16_t*>(a.q)[at] = hi;
            static_cast<uint16_t*>(a.q)[(int64_t)a.heads * row + at] = f_bf16(v - bf16_f(hi));
        } else {
            static_cast<float*>(a.q)[at] = v;
        }
    };
    if (tid < 128 && r0 + tid < rank8) {
        float v = 0.0f;
#pragma unroll
        for (int k = 0; k < 16; ++k) v += s_sum[k][tid];
        put_q(r0 + tid, v);  // columns past kv_rank hold zero weights
    }
    if (r0 == 0)
        for (int i = tid; i < rot8; i += 256) {
            float v = 0.0f;
            if (i < a.rot_dim) {
                v = q[a.dim + i];
                if (i < 2 * half) {
                    const float c = cs[2 * (i >> 1)], sn = cs[2 * (i >> 1) + 1], o = q[a.dim + (i ^ 1)];
                    v = (i & 1) ? v * c + o * sn : v * c - o * sn;
                }
            }
            put_q(rank8 + i, v);
        }
}

int latent_absorb(const LatentStep& a, hipStream_t s) {
    if (a.dim > 1024) return PTM_E_UNSUPPORTED;
    const dim3 grid(a.heads * ((a.kv_rank + 127) / 128) + 1);
    if (a.fp32) hipLaunchKernelGGL(latent_absorb_kernel<true>, grid, dim3(256), 0, s, a);
    else hipLaunchKernelGGL(latent_absorb_kernel<false>, grid, dim3(256), 0, s, a);
    return launch_status();
}

// grid (heads, ceil(vdim / 32)).  The head's split results are merged into its latent (LDS), which 32 rows of W_uv take to
// the head's output: 8 rows per wave, their first 512 columns requested before the merge.
constexpr int LO_MAX_SPLITS = 256;
__global__ __launch_bounds__(256) void latent_out_kernel(const uint16_t* __restrict__ w_uv, int64_t ld, int heads, int kv_rank,
                                                         int vdim, const float* __restrict__ pO, const float* __restrict__ pM,
                                                         const float* __restrict__ pL, int splits, int o_row,
                                                         float* __restrict__ out) {
    extern __shared__ __align__(16) float s_c[];  // [up64(kv_rank)]
    __shared__ float s_w[LO_MAX_SPLITS];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int h = blockIdx.x, v8 = (vdim + 7) & ~7, kp = (kv_rank + 63) & ~63;
    const int v0 = blockIdx.y * 32 + wave * 8;
    const uint16_t* w = w_uv + (int64_t)h * v8 * ld;
    u32x4 wr[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) {
        wr[i] = u32x4{0, 0, 0, 0};
        if (lane * 8 < kp) wr[i] = *reinterpret_cast<const u32x4*>(w + (int64_t)min(v0 + i, vdim - 1) * ld + lane * 8);
    }
    issue_order_fence();
    // the first 512 latent values of up to 24 splits are requested before the weights are known
    float2 pre[24];
    {
        const float* p = pO + (int64_t)h * o_row + min(tid * 2, o_row - 2);
#pragma unroll
        for (int i = 0; i < 24; ++i) pre[i] = *reinterpret_cast<const float2*>(p + (int64_t)min(i, splits - 1) * heads * o_row);
    }
    issue_order_fence();
    if (pM) {
        if (wave == 0) {
            float mv[LO_MAX_SPLITS / 64], lv[LO_MAX_SPLITS / 64], m = -INFINITY;
#pragma unroll
            for (int u = 0; u < LO_MAX_SPLITS / 64; ++u) {
                const int i = min(lane + 64 * u, splits - 1);
                mv[u] = lane + 64 * u < splits ? pM[(int64_t)i * heads + h] : -INFINITY;
                lv[u] = pL[(int64_t)i * heads + h];
                m = fmaxf(m, mv[u]);
            }
            m = max64(m);
            float l = 0.0f;
#pragma unroll
            for (int u = 0; u < LO_MAX_SPLITS / 64; ++u) {
                mv[u] = expf(mv[u] - m);
                l = fmaf(lv[u], mv[u], l);
            }
            l = 1.0f / sum64(l);
#pragma unroll
            for (int u = 0; u < LO_MAX_SPLITS / 64; ++u) s_w[lane + 64 * u] = mv[u] * l;  // 0 past the last split
        }
    } else if (tid < 64) {
        s_w[tid] = tid == 0 ? 1.0f : 0.0f;
    }
    __syncthreads();
    for (int r = tid * 2; r < kp; r += 512) {
        float a0 = 0.0f, a1 = 0.0f;
        if (r < kv_rank) {
            const float* p = pO + (int64_t)h * o_row + r;
            int i = 0;
            if (r < 512) {
#pragma unroll
                for (int k = 0; k < 24; ++k) {
                    a0 = fmaf(pre[k].x, s_w[k], a0);
                    a1 = fmaf(pre[k].y, s_w[k], a1);
                }
                i = 24;
            }
#pragma unroll 8
            for (; i < splits; ++i) {  // a share without a visible key has weight 0
                const float2 v = *reinterpret_cast<const float2*>(p + (int64_t)i * heads * o_row);
                a0 = fmaf(v.x, s_w[i], a0);
                a1 = fmaf(v.y, s_w[i], a1);
            }
        }
        s_c[r] = a0;
        s_c[r + 1] = r + 1 < kv_rank ? a1 : 0.0f;
    }
    __syncthreads();
    float acc[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) acc[i] = 0.0f;
    for (int k = lane * 8; k < kp; k += 512) {
        if (k >= 512)
#pragma unroll
            for (int i = 0; i < 8; ++i) wr[i] = *reinterpret_cast<const u32x4*>(w + (int64_t)min(v0 + i, vdim - 1) * ld + k);
        const float4 x0 = *reinterpret_cast<const float4*>(s_c + k), x1 = *reinterpret_cast<const float4*>(s_c + k + 4);
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            float t = acc[i];
            t = fmaf(bf16_lo(wr[i].x), x0.x, t);
            t = fmaf(bf16_hi(wr[i].x), x0.y, t);
            t = fmaf(bf16_lo(wr[i].y), x0.z, t);
            t = fmaf(bf16_hi(wr[i].y), x0.w, t);
            t = fmaf(bf16_lo(wr[i].z), x1.x, t);
            t = fmaf(bf16_hi(wr[i].z), x1.y, t);
            t = fmaf(bf16_lo(wr[i].w), x1.z, t);
            t = fmaf(bf16_hi(wr[i].w), x1.w, t);
            acc[i] = t;
        }
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) {
        const float s = sum64(acc[i]);
        if (lane == 0 && v0 + i < vdim) out[(int64_t)h * v8 + v0 + i] = s;
    }
}

int latent_out(const LatentStep& a, const float* pO, const float* pM, const float* pL, int splits, int o_row, float* out,
               hipStream_t s) {
    if (splits > LO_MAX_SPLITS || a.kv_rank > 8192) return PTM_E_UNSUPPORTED;
    const uint16_t* w_uv = a.expand + (int64_t)a.heads * up8(a.dim) * a.ld;
    hipLaunchKernelGGL(latent_out_kernel, dim3(a.heads, (a.vdim + 31) / 32), dim3(256), (size_t)up64(a.kv_rank) * 4, s, w_uv, a.ld,
                       a.heads, a.kv_rank, a.vdim, pO, pM, pL, splits, o_row, out);
    return launch_status();
}

}  // namespace ptm

extern "C" int ptm_dense_cols(int cols) { return ptm::up64(cols); }

extern "C" int ptm_dense_gemv(const void* W, const float* x, float* y, int K, int N, int64_t ld, ptm_stream_t stream) {
    if (!W || !x || !y) return PTM_E_NULL;
    if ((size_t)ptm::up64(K) * 4 > 64 * 1024) ptm::dense_gemv_init();
    ptm::DenseGemv g;
    g.W = static_cast<const uint16_t*>(W);
    g.ld = ld;
    g.N = N;
    g.K = K;
    g.x = x;
    g.y = y;
    return ptm::dense_gemv(g, ptm::as_stream(stream));
}
