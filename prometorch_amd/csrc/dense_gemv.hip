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

// A vector formed from streams, in LDS: blend of the streams and the pending branch, norm, token shift.  sec: section of the
// workgroup's rows.  PUT(i, v) / GET(i): float4 i of the vector.
template <typename Put, typename Get>
__device__ __forceinline__ void stream_prologue(const DenseGemv& a, int sec, float* red, Put put, Get get) {
    const int tid = threadIdx.x, Kp = (a.K + 63) & ~63, n4 = Kp / 4, S = a.streams;
    const bool first = blockIdx.x == 0;
    float mean = 0.0f;
    float4 prev[2][2];  // both ring slots of the first two pieces, requested before the position is known
    const int64_t pos = a.mu ? *a.d_past : 0;
    if (a.mu) {
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int z = 0; z < 2; ++z) prev[u][z] = ld4(a.shift + (int64_t)z * Kp, min(tid + u * DG_THREADS, n4 - 1));
    }
    auto mix = [&](int i, const float* c) {
        float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll 4
        for (int t = 0; t < S; ++t) {
            const float4 x = ld4(a.x + t * a.x_stride, i);
            const float b = c[t];
            v = make_float4(fmaf(b, x.x, v.x), fmaf(b, x.y, v.y), fmaf(b, x.z, v.z), fmaf(b, x.w, v.w));
        }
        if (a.h) {
            const float4 x = ld4(a.h, i);
            const float b = c[S];
            v = make_float4(fmaf(b, x.x, v.x), fmaf(b, x.y, v.y), fmaf(b, x.z, v.z), fmaf(b, x.w, v.w));
        }
        return v;
    };
    float sum = 0.0f;
#pragma unroll 2
    for (int i = tid; i < n4; i += DG_THREADS) {
        const float4 v = mix(i, a.blend);
        sum += (v.x + v.y) + (v.z + v.w);
        put(i, v);
    }
    if (a.h && a.store)  // the new streams
        for (int t = blockIdx.x; t < S; t += gridDim.x)
            for (int i = tid; i < n4; i += DG_THREADS) reinterpret_cast<float4*>(a.xout + (int64_t)t * Kp)[i] = mix(i, a.store + (int64_t)t * (S + 1));
    if (!a.gamma && !a.mu) return;
    if (a.beta) mean = block_sum<DG_WAVES>(sum, red) / (float)a.K;
    auto centred = [&](int i, float4 v) {  // padding is not part of the variance
        v = make_float4(v.x - mean, v.y - mean, v.z - mean, v.w - mean);
        if (4 * i + 3 >= a.K) {
            if (4 * i >= a.K) v.x = 0.0f;
            if (4 * i + 1 >= a.K) v.y = 0.0f;
            if (4 * i + 2 >= a.K) v.z = 0.0f;
            v.w = 0.0f;
        }
        return v;
    };
    float r = 1.0f;
    if (a.gamma) {
        float ss = 0.0f;
        for (int i = tid; i < n4; i += DG_THREADS) ss = sq4(centred(i, get(i)), ss);  // a thread reads the pieces it wrote itself
        r = 1.0f / sqrtf(block_sum<DG_WAVES>(ss, red) / (float)a.K + a.eps);
    }
    auto finish = [&](int i, float4 p) {
        float4 v = get(i);
        if (a.gamma) {
            const float4 g = ld4(a.gamma, i);
            v = centred(i, v);
            v = make_float4(v.x * r * g.x, v.y * r * g.y, v.z * r * g.z, v.w * r * g.w);
            if (a.beta) v = add4(v, ld4(a.beta, i));
        }
        if (first && a.xn_out) reinterpret_cast<float4*>(a.xn_out)[i] = v;
        if (a.mu) {
            if (first) reinterpret_cast<float4*>(a.shift + (pos & 1) * Kp)[i] = v;
            if (pos == 0) p = make_float4(0.f, 0.f, 0.f, 0.f);
            const float4 m = ld4(a.mu + (int64_t)sec * Kp, i);
            v = make_float4(fmaf(p.x - v.x, m.x, v.x), fmaf(p.y - v.y, m.y, v.y), fmaf(p.z - v.z, m.z, v.z), fmaf(p.w - v.w, m.w, v.w));
        }
        put(i, v);
    };
#pragma unroll
    for (int u = 0; u < 2; ++u) {
        const int i = tid + u * DG_THREADS;
        if (i < n4) finish(i, a.mu ? (pos & 1) ? prev[u][0] : prev[u][1] : make_float4(0.f, 0.f, 0.f, 0.f));
    }
    for (int i = tid + 2 * DG_THREADS; i < n4; i += DG_THREADS)
        finish(i, a.mu ? ld4(a.shift + ((pos & 1) ^ 1) * Kp, i) : make_float4(0.f, 0.f, 0.f, 0.f));
}

// The vector with its tail normed in equal parts; s_r: one float per part.  AT(e): element e of the vector in LDS.
template <typename Put, typename At>
__device__ __forceinline__ void tail_prologue(const DenseGemv& a, float* s_r, float* red, Put put, At at) {
    const int tid = threadIdx.x, Kp = (a.K + 63) & ~63, n4 = Kp / 4, part = a.tail_n / a.tail_parts;
    for (int i = tid; i < n4; i += DG_THREADS) put(i, ld4(a.x, i));
    __syncthreads();
    if (a.tail_parts <= 4) {
        for (int p = 0; p < a.tail_parts; ++p) {
            float ss = 0.0f;
            for (int e = tid; e < part; e += DG_THREADS) {
                const float v = *at(a.tail0 + p * part + e);
                ss = fmaf(v, v, ss);
            }
            ss = block_sum<DG_WAVES>(ss, red);
            if (tid == 0) s_r[p] = 1.0f / sqrtf(ss / (float)part + a.eps);
        }
    } else {
        for (int p = tid >> 6; p < a.tail_parts; p += DG_WAVES) {
            float ss = 0.0f;
            for (int e = tid & 63; e < part; e += 64) {
                const float v = *at(a.tail0 + p * part + e);
                ss = fmaf(v, v, ss);
            }
            ss = sum64(ss);
            if ((tid & 63) == 0) s_r[p] = 1.0f / sqrtf(ss / (float)part + a.eps);
        }
    }
    __syncthreads();
    for (int e = tid; e < a.tail_n; e += DG_THREADS) {
        float* v = at(a.tail0 + e);
        *v = *v * s_r[e / part] * a.tail_norm[e] * a.tail_scale;
    }
}

// PRO: what forms the vector - 0: nothing, 1: residual and RMS norm, 2: streams, 3: the tail's norm
template <int LPR, int R, int U, int PRO, bool GLU>
__global__ __launch_bounds__(DG_THREADS, 4) void dense_gemv_kernel(const DenseGemv a) {
    static_assert(!GLU || R % 2 == 0, "a lane holds the gate and the up row of a value");
    extern __shared__ __align__(16) float4 s_x[];  // [2][Kp / 8]
    __shared__ float red[DG_WAVES];
    __shared__ int redi[DG_WAVES];
    constexpr int RPP = 64 / LPR, RW = GLU ? RPP * R / 2 : RPP * R;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int li = lane % LPR, lr = lane / LPR;
    const int Kp = (a.K + 63) & ~63, n4 = Kp / 4, n8 = Kp / 8;
    int sec = 0, row0 = 0, rows = a.N, wg = blockIdx.x, wgs = gridDim.x;
    if constexpr (PRO == 2) {
        if (a.sections > 0) {
            while (sec + 1 < a.sections && wg >= a.section_wg[sec + 1]) ++sec;
            wg -= a.section_wg[sec];
            wgs = a.section_wg[sec + 1] - a.section_wg[sec];
            row0 = a.section_row[sec];
            rows = a.section_row[sec + 1] - row0;
        }
    }
    const int groups = (rows + RW - 1) / RW, stride = wgs * DG_WAVES;
    const int nb = (n8 + LPR * U - 1) / (LPR * U);
    const uint32_t bytes = (uint32_t)((int64_t)a.N * a.ld * (GLU ? 4 : 2));
    const __amdgpu_buffer_rsrc_t rs = make_rsrc(a.W, (int)bytes);
    auto load = [&](int g, int b, u32x4* w) {
#pragma unroll
        for (int r = 0; r < R; ++r) {
            int row;
            if constexpr (GLU) row = min(g * RW + r / 2 * RPP + lr, rows - 1) + (r & 1) * rows;
            else row = row0 + min(g * RW + r * RPP + lr, rows - 1);
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
    int g = wg * DG_WAVES + wave, b = 0;
    auto at = [&](int e) { return reinterpret_cast<float*>(s_x + ((e >> 2) & 1) * n8 + (e >> 3)) + (e & 3); };
    if constexpr (PRO == 2) {
        load(min(g, groups - 1), 0, cur);
        issue_order_fence();
        stream_prologue(a, sec, red, put, [&](int i) { return s_x[(i & 1) * n8 + (i >> 1)]; });
        __syncthreads();
    } else if constexpr (PRO == 3) {
        load(min(g, groups - 1), 0, cur);
        issue_order_fence();
        tail_prologue(a, reinterpret_cast<float*>(s_x + 2 * n8), red, put, at);
        __syncthreads();
    } else if constexpr (PRO == 0) {
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
    float acc[R], glu_gate = 0.0f;
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
                if constexpr (GLU) {
                    const int pair = g * RW + r / 2 * RPP + lr;
                    if (r & 1) {
                        if (li == 0 && pair < rows) a.y[pair] = glu_gate * v;
                    } else {
                        glu_gate = silu_f(v);
                    }
                    continue;
                }
                const int row = row0 + g * RW + r * RPP + lr;
                if (li == 0 && row < row0 + rows) {
                    v *= a.out_scale;
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
    const bool glu = g.epilogue == GEMV_SWIGLU;
    if (kp <= 64) return {0, glu ? 16 : 32};
    if (kp <= 256) return {1, glu ? 4 : 8};
    if (glu) return ch <= 2 ? GemvShape{2, 2} : GemvShape{3, 1};
    const bool few = g.N <= 2 * DG_WAVES * 256;  // two rows per wave would leave compute units without work
    if (ch <= 2) return few ? GemvShape{5, 1} : GemvShape{2, 4};
    if (ch <= 4 || (ch <= 7 && !few)) return few ? GemvShape{5, 1} : GemvShape{3, 2};
    return {4, 1};
}
// At most 512 workgroups (one more would run by itself behind the others): as many as its rows fill for a section of few rows,
// the rest over the others by their rows.
void section_workgroups(DenseGemv& g) {
    const int per = gemv_shape(g).rows_per_wave * DG_WAVES;
    int64_t room = 512, rows_left = 0;
    auto rows = [&](int i) { return (int64_t)(g.section_row[i + 1] - g.section_row[i]); };
    auto fill = [&](int i) { return (rows(i) + per - 1) / per; };
    auto small = [&](int i) { return rows(i) * 16 < g.N && fill(i) <= 16; };
    for (int i = 0; i < g.sections; ++i) {
        if (small(i)) room -= fill(i);
        else rows_left += rows(i);
    }
    for (int i = 0; i < g.sections; ++i) {
        int64_t n = fill(i);
        if (!small(i) && n > room * rows(i) / rows_left) n = room * rows(i) / rows_left;
        g.section_wg[i + 1] = g.section_wg[i] + (int)(n > 0 ? n : 1);
    }
}
}  // namespace

int dense_gemv_workgroups(const DenseGemv& g) {
    const int groups = (g.N + gemv_shape(g).rows_per_wave - 1) / gemv_shape(g).rows_per_wave;
    const int wgs = (groups + DG_WAVES - 1) / DG_WAVES;
    return wgs < 512 ? wgs : 512;
}

template <int PRO>
static void gemv_attr() {
    const int lds = 150 * 1024;
#define PTM_DG(...) (void)hipFuncSetAttribute(reinterpret_cast<const void*>(dense_gemv_kernel<__VA_ARGS__>), hipFuncAttributeMaxDynamicSharedMemorySize, lds)
    PTM_DG(8, 4, 1, PRO, false);
    PTM_DG(32, 4, 1, PRO, false);
    PTM_DG(64, 4, 2, PRO, false);
    PTM_DG(64, 2, 4, PRO, false);
    PTM_DG(64, 1, 8, PRO, false);
    PTM_DG(64, 1, 4, PRO, false);
    if constexpr (PRO < 3) {
        PTM_DG(8, 4, 1, PRO, true);
        PTM_DG(32, 4, 1, PRO, true);
        PTM_DG(64, 4, 2, PRO, true);
        PTM_DG(64, 2, 4, PRO, true);
    }
#undef PTM_DG
}
// one-time kernel attributes, before anything can be captured
void dense_gemv_init() {
    gemv_attr<0>();
    gemv_attr<1>();
    gemv_attr<2>();
    gemv_attr<3>();
}

template <int PRO>
static void gemv_launch(const DenseGemv& g, dim3 grid, size_t lds, hipStream_t s) {
    const dim3 block(DG_THREADS);
#define PTM_DG(...) hipLaunchKernelGGL((dense_gemv_kernel<__VA_ARGS__>), grid, block, lds, s, g)
    if constexpr (PRO < 3) {
        if (g.epilogue == GEMV_SWIGLU) {
            switch (gemv_shape(g).kind) {
                case 0: PTM_DG(8, 4, 1, PRO, true); break;
                case 1: PTM_DG(32, 4, 1, PRO, true); break;
                case 2: PTM_DG(64, 4, 2, PRO, true); break;
                default: PTM_DG(64, 2, 4, PRO, true); break;
            }
            return;
        }
    }
    switch (gemv_shape(g).kind) {
        case 0: PTM_DG(8, 4, 1, PRO, false); break;
        case 1: PTM_DG(32, 4, 1, PRO, false); break;
        case 2: PTM_DG(64, 4, 2, PRO, false); break;
        case 3: PTM_DG(64, 2, 4, PRO, false); break;
        case 4: PTM_DG(64, 1, 8, PRO, false); break;
        default: PTM_DG(64, 1, 4, PRO, false); break;
    }
#undef PTM_DG
}

int dense_gemv(DenseGemv g, hipStream_t s) {
    if (!g.W || !g.x || !g.y) return PTM_E_NULL;
    if (g.N <= 0 || g.K <= 0 || g.ld < up64(g.K)) return PTM_E_SHAPE;
    const int64_t rows = g.epilogue == GEMV_SWIGLU ? 2 * (int64_t)g.N : g.N;
    if (up64(g.K) > 36864 || rows * g.ld * 2 >= (int64_t)0xfffffff0u) return PTM_E_UNSUPPORTED;
    if (!aligned16(g.W) || !aligned16(g.x) || (g.ld & 7)) return PTM_E_ALIGN;
    if (g.sections > 0) {
        if (g.sections > GEMV_SECTIONS || g.streams <= 0 || g.section_row[0] != 0 || g.section_row[g.sections] != g.N) return PTM_E_SHAPE;
        for (int i = 0; i < g.sections; ++i)
            if (g.section_row[i + 1] <= g.section_row[i]) return PTM_E_SHAPE;
        section_workgroups(g);
    }
    const dim3 grid(g.sections > 0 ? g.section_wg[g.sections] : dense_gemv_workgroups(g));
    const size_t lds = (size_t)up64(g.K) * 4;
    if (g.streams > 0) {
        if (!g.blend || (g.store && !g.xout) || (g.mu && (!g.shift || !g.d_past)) || (g.beta && !g.gamma)) return PTM_E_NULL;
        if (g.x_stride & 3) return PTM_E_ALIGN;
        gemv_launch<2>(g, grid, lds, s);
    } else if (g.tail_n > 0) {
        if (!g.tail_norm) return PTM_E_NULL;
        if (g.tail_parts <= 0 || g.tail_n % g.tail_parts || g.tail0 + g.tail_n > g.K) return PTM_E_SHAPE;
        if (g.epilogue == GEMV_SWIGLU || g.tail_parts > 512) return PTM_E_UNSUPPORTED;
        gemv_launch<3>(g, grid, lds + (size_t)g.tail_parts * 4, s);
    } else if (g.h || g.add0 || g.add1 || g.gamma || g.xout || g.xn_out) {
        gemv_launch<1>(g, grid, lds, s);
    } else {
        gemv_launch<0>(g, grid, lds, s);
    }
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
