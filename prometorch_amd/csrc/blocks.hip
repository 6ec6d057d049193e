// Layers of a block decoder: the token step and the prompt rows over a list of blocks with a mixer each, a loop of blocks
// with shared weights, and a per-layer token input.  The residual, the norms, rotations, scores and softmax are fp32.
//
// Token step, launches per layer (the post-norm and residual add of a branch wait in `pend` for the next projection's
// prologue, which also takes in what a loop pass adds):
//   attention  [post-norm + norm1 + q|k|v]  [qk-norm + rotation + append + split attention]  [merge]  [out]
//   latent     [post-norm + norm1 + q|c]    [W_uk onto q + rotation + latent norm + append]  [split attention]  [merge + W_uv]  [out]
//   both       [post-norm + norm2 + up + relu^2]  [down]  [post-norm + gate + gelu * e]  [proj]
// With streams (hyper-connections) the pending part is a branch output and its blend weights: the next projection's prologue forms
// the blend it reads straight from the old streams, and its first workgroups store the new ones.
//   wkv        [streams + norm1 + token shift + r|k|v|g|w1]  [w2 + state + head norm + gate]  [out]
//   attention and state-space side by side
//              [streams + norm1 + q|k|v|g|z|x|B|C|dt]  [qk-norm + append + split attention]  [merge + sink + gate]
//              [convolution + state]  [state-space norm + out]
//   swiglu     [streams + norm2 + gate, up + silu]  [down]
// Prompt rows: the same with one GEMM per projection (activation and token input in its epilogue) and one row launch per norm.
#include "blocks.h"

#include <cmath>
#include <new>
#include <vector>

namespace ptm {

// ---- row kernels ------------------------------------------------------------------------------
// grid (rows, wp / 512): out[r][:] = table row of tokens[r] (the table's rows are padded like the output's)
__global__ __launch_bounds__(128) void embed_bf16_rows_kernel(const uint16_t* __restrict__ table, int64_t ld, const int* __restrict__ tokens,
                                                              int wp, float* __restrict__ out, float* __restrict__ out2) {
    const int i = (blockIdx.y * 128 + threadIdx.x) * 4;
    if (i >= wp) return;
    const uint2 u = *reinterpret_cast<const uint2*>(table + (int64_t)tokens[blockIdx.x] * ld + i);
    const float4 v = make_float4(bf16_lo(u.x), bf16_hi(u.x), bf16_lo(u.y), bf16_hi(u.y));
    *reinterpret_cast<float4*>(out + (int64_t)blockIdx.x * wp + i) = v;
    if (out2) *reinterpret_cast<float4*>(out2 + (int64_t)blockIdx.x * wp + i) = v;
}

// grid rows: x += RMS(h) * hw + add0 + add1 (each optional), then xn = RMS(x) * gamma (gamma NULL: xn = x; xn NULL: nothing).
// h may still be `slabs` partial sums, `slab` floats apart.
template <bool F32>
__global__ __launch_bounds__(256) void residual_norm_rows_kernel(float* __restrict__ x, const float* __restrict__ h,
                                                                 int slabs, int64_t slab, const float* __restrict__ hw,
                                                                 const float* __restrict__ add0, const float* __restrict__ add1,
                                                                 const float* __restrict__ gamma, void* __restrict__ xn, int hidden, int wp, float eps) {
    __shared__ float red[4];
    const int64_t base = (int64_t)blockIdx.x * wp;
    float4* x4 = reinterpret_cast<float4*>(x + base);
    const float4* h4 = reinterpret_cast<const float4*>(h + base);
    const float4* a4 = reinterpret_cast<const float4*>(add0 + base);
    const int n4 = wp / 4;
    auto h_at = [&](int i) {
        float4 v = h4[i];
#pragma unroll 5
        for (int z = 1; z < slabs; ++z) {
            const float4 p = *reinterpret_cast<const float4*>(h + base + z * slab + 4 * i);
            v = make_float4(v.x + p.x, v.y + p.y, v.z + p.z, v.w + p.w);
        }
        if (4 * i + 3 >= hidden) {  // the slabs' padding is not kept clear
            if (4 * i >= hidden) v.x = 0.0f;
            if (4 * i + 1 >= hidden) v.y = 0.0f;
            if (4 * i + 2 >= hidden) v.z = 0.0f;
            v.w = 4 * i + 3 >= hidden ? 0.0f : v.w;
        }
        return v;
    };
    constexpr int NS = 8;  // slots kept in registers: rows of up to 8192 values are read once
    float4 xv[NS], hv[NS];
    float rh = 0.0f;
    if (h) {
        float ss = 0.0f;
#pragma unroll
        for (int u = 0; u < NS; ++u) {
            const int i = threadIdx.x + 256 * u;
            hv[u] = i < n4 ? h_at(i) : make_float4(0.f, 0.f, 0.f, 0.f);
            ss = fmaf(hv[u].x, hv[u].x, fmaf(hv[u].y, hv[u].y, fmaf(hv[u].z, hv[u].z, fmaf(hv[u].w, hv[u].w, ss))));
        }
        for (int i = threadIdx.x + 256 * NS; i < n4; i += 256) {
            const float4 v = h_at(i);
            ss = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, ss))));
        }
        rh = 1.0f / sqrtf(block_sum<4>(ss, red) / (float)hidden + eps);
    }
    const float4* w4 = reinterpret_cast<const float4*>(hw);
    const float4* b4 = reinterpret_cast<const float4*>(add1);
    auto combine = [&](int i, float4 v, float4 hh) {
        if (h) {
            const float4 w = w4[i];
            v = make_float4(v.x + hh.x * rh * w.x, v.y + hh.y * rh * w.y, v.z + hh.z * rh * w.z, v.w + hh.w * rh * w.w);
        }
        if (add0) { const float4 a = a4[i]; v = make_float4(v.x + a.x, v.y + a.y, v.z + a.z, v.w + a.w); }
        if (add1) { const float4 a = b4[i]; v = make_float4(v.x + a.x, v.y + a.y, v.z + a.z, v.w + a.w); }
        return v;
    };
    const bool changed = h || add0 || add1;
    float ss = 0.0f;
#pragma unroll
    for (int u = 0; u < NS; ++u) {
        const int i = threadIdx.x + 256 * u;
        xv[u] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (i < n4) {
            xv[u] = combine(i, x4[i], hv[u]);
            if (changed) x4[i] = xv[u];
        }
        ss = fmaf(xv[u].x, xv[u].x, fmaf(xv[u].y, xv[u].y, fmaf(xv[u].z, xv[u].z, fmaf(xv[u].w, xv[u].w, ss))));
    }
    for (int i = threadIdx.x + 256 * NS; i < n4; i += 256) {
        const float4 v = combine(i, x4[i], h ? h_at(i) : make_float4(0.f, 0.f, 0.f, 0.f));
        if (changed) x4[i] = v;
        ss = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, ss))));
    }
    if (!xn) return;
    float r = 1.0f;
    if (gamma) r = 1.0f / sqrtf(block_sum<4>(ss, red) / (float)hidden + eps);
    const float4* g4 = reinterpret_cast<const float4*>(gamma);
    auto emit = [&](int i, float4 v) {
        if (gamma) {
            const float4 g = g4[i];
            v = make_float4(v.x * r * g.x, v.y * r * g.y, v.z * r * g.z, v.w * r * g.w);
        }
        if constexpr (F32) {
            *reinterpret_cast<float4*>(static_cast<float*>(xn) + base + 4 * i) = v;
        } else {
            *reinterpret_cast<uint2*>(static_cast<uint16_t*>(xn) + base + 4 * i) =
                make_uint2((uint32_t)f_bf16(v.x) | ((uint32_t)f_bf16(v.y) << 16), (uint32_t)f_bf16(v.z) | ((uint32_t)f_bf16(v.w) << 16));
        }
    };
#pragma unroll
    for (int u = 0; u < NS; ++u) {
        const int i = threadIdx.x + 256 * u;
        if (i < n4) emit(i, xv[u]);
    }
    for (int i = threadIdx.x + 256 * NS; i < n4; i += 256) emit(i, x4[i]);  // a thread reads back what it stored itself
}

// grid rows: compact copy of the residual rows (the sum of their streams)
__global__ __launch_bounds__(256) void copy_rows_kernel(const float* __restrict__ x, int streams, int64_t stride, int wp, int hidden, float* __restrict__ out) {
    for (int i = threadIdx.x; i < hidden; i += 256) {
        float v = x[(int64_t)blockIdx.x * wp + i];
        for (int t = 1; t < streams; ++t) v += x[t * stride + (int64_t)blockIdx.x * wp + i];
        out[(int64_t)blockIdx.x * hidden + i] = v;
    }
}

// grid (rows, wp / 512): `streams` copies, `stride` floats apart, of the token's table row plus (freq given) the sinusoid of its
// position: pair i turns by position * freq[i], sin first.  Angles in double up to a turn.
__global__ __launch_bounds__(128) void embed_streams_kernel(const uint16_t* __restrict__ table, int64_t ld, const int* __restrict__ tokens,
                                                            const double* __restrict__ freq, const int64_t* __restrict__ d_past, int64_t pos0,
                                                            int hidden, int wp, int streams, int64_t stride, float* __restrict__ out) {
    const int i = (blockIdx.y * 128 + threadIdx.x) * 4;
    if (i >= wp) return;
    const uint2 u = *reinterpret_cast<const uint2*>(table + (int64_t)tokens[blockIdx.x] * ld + i);
    float4 v = make_float4(bf16_lo(u.x), bf16_hi(u.x), bf16_lo(u.y), bf16_hi(u.y));
    if (freq) {
        const double p = (double)((d_past ? *d_past : pos0) + blockIdx.x), turn = 6.283185307179586476925;
        auto angle = [&](int k) {
            const double a = p * freq[k];
            return (float)(a - turn * rint(a / turn));
        };
        const float a0 = angle(i / 2), a1 = angle(i / 2 + 1);
        if (i < hidden) v.x += sinf(a0);
        if (i + 1 < hidden) v.y += cosf(a0);
        if (i + 2 < hidden) v.z += sinf(a1);
        if (i + 3 < hidden) v.w += cosf(a1);
    }
    for (int t = 0; t < streams; ++t) *reinterpret_cast<float4*>(out + t * stride + (int64_t)blockIdx.x * wp + i) = v;
}

struct StreamRows {
    float* x;              // [streams], stride floats apart, of rows of wp
    int streams;
    int64_t stride;
    const float* h;        // pending branch output (NULL: none), `slabs` partial sums, `slab` floats apart
    int slabs;
    int64_t slab;
    const float* store;    // [streams][streams + 1]: the new streams
    const float* blend;    // [streams]: the vector that is normed, from the new streams
    const float *gamma, *beta;
    void* xn;              // NULL: only the streams
    int hidden, wp;
    float eps;
};
// grid rows: x_t <- sum_s store[t][s] x_s + store[t][streams] h, then xn = norm(sum_t blend[t] x_t).  Up to MAXS streams.
template <bool F32, int MAXS>
__global__ __launch_bounds__(256) void stream_norm_rows_kernel(const StreamRows a) {
    __shared__ float red[4];
    __shared__ float s_c[MAXS * (MAXS + 1) + MAXS];
    const int64_t base = (int64_t)blockIdx.x * a.wp;
    const int n4 = a.wp / 4, S = a.streams;
    if (a.h)
        for (int i = threadIdx.x; i < S * (S + 1); i += 256) s_c[i] = a.store[i];
    if (a.xn)
        for (int i = threadIdx.x; i < S; i += 256) s_c[MAXS * (MAXS + 1) + i] = a.blend[i];
    __syncthreads();
    auto mul = [](float4 v, float4 x, float c) { return make_float4(fmaf(c, x.x, v.x), fmaf(c, x.y, v.y), fmaf(c, x.z, v.z), fmaf(c, x.w, v.w)); };
    auto h_at = [&](int i) {
        float4 v = *reinterpret_cast<const float4*>(a.h + base + 4 * i);
#pragma unroll 4
        for (int z = 1; z < a.slabs; ++z) {
            const float4 p = *reinterpret_cast<const float4*>(a.h + base + z * a.slab + 4 * i);
            v = make_float4(v.x + p.x, v.y + p.y, v.z + p.z, v.w + p.w);
        }
        if (4 * i + 3 >= a.hidden) {  // the slabs' padding is not kept clear
            if (4 * i >= a.hidden) v.x = 0.0f;
            if (4 * i + 1 >= a.hidden) v.y = 0.0f;
            if (4 * i + 2 >= a.hidden) v.z = 0.0f;
            v.w = 0.0f;
        }
        return v;
    };
    // streams of float4 i updated; returns their blend
    auto advance = [&](int i) {
        float4 xs[MAXS], u = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int t = 0; t < MAXS; ++t)
            if (t < S) xs[t] = *reinterpret_cast<const float4*>(a.x + t * a.stride + base + 4 * i);
        if (a.h) {
            const float4 h = h_at(i);
#pragma unroll
            for (int t = 0; t < MAXS; ++t) {
                if (t >= S) break;
                const float* c = s_c + t * (S + 1);
                float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
                for (int q = 0; q < MAXS; ++q)
                    if (q < S) v = mul(v, xs[q], c[q]);
                v = mul(v, h, c[S]);
                *reinterpret_cast<float4*>(a.x + t * a.stride + base + 4 * i) = v;
                if (a.xn) u = mul(u, v, s_c[MAXS * (MAXS + 1) + t]);
            }
        } else if (a.xn) {
#pragma unroll
            for (int t = 0; t < MAXS; ++t)
                if (t < S) u = mul(u, xs[t], s_c[MAXS * (MAXS + 1) + t]);
        }
        return u;
    };
    auto centred = [&](int i, float4 v, float mean) {
        v = make_float4(v.x - mean, v.y - mean, v.z - mean, v.w - mean);
        if (4 * i + 3 >= a.hidden) {
            if (4 * i >= a.hidden) v.x = 0.0f;
            if (4 * i + 1 >= a.hidden) v.y = 0.0f;
            if (4 * i + 2 >= a.hidden) v.z = 0.0f;
            v.w = 0.0f;
        }
        return v;
    };
    // the blend of the streams as they are now (longer rows than the registers hold)
    auto again = [&](int i) {
        float4 u = make_float4(0.f, 0.f, 0.f, 0.f);
        for (int t = 0; t < S; ++t) u = mul(u, *reinterpret_cast<const float4*>(a.x + t * a.stride + base + 4 * i), s_c[MAXS * (MAXS + 1) + t]);
        return u;
    };
    constexpr int NS = 4;
    float4 uv[NS];
    float sum = 0.0f;
#pragma unroll
    for (int k = 0; k < NS; ++k) {
        const int i = threadIdx.x + 256 * k;
        uv[k] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (i < n4) uv[k] = advance(i);
        sum += (uv[k].x + uv[k].y) + (uv[k].z + uv[k].w);
    }
    for (int i = threadIdx.x + 256 * NS; i < n4; i += 256) {
        const float4 v = advance(i);
        sum += (v.x + v.y) + (v.z + v.w);
    }
    if (!a.xn) return;
    const float mean = a.beta ? block_sum<4>(sum, red) / (float)a.hidden : 0.0f;
    auto sq = [](float4 v, float s) { return fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, s)))); };
    float ss = 0.0f;
#pragma unroll
    for (int k = 0; k < NS; ++k) {
        const int i = threadIdx.x + 256 * k;
        if (i < n4) {
            uv[k] = centred(i, uv[k], mean);
            ss = sq(uv[k], ss);
        }
    }
    for (int i = threadIdx.x + 256 * NS; i < n4; i += 256) ss = sq(centred(i, again(i), mean), ss);
    const float r = 1.0f / sqrtf(block_sum<4>(ss, red) / (float)a.hidden + a.eps);
    auto emit = [&](int i, float4 v) {
        const float4 g = reinterpret_cast<const float4*>(a.gamma)[i];
        float4 b = make_float4(0.f, 0.f, 0.f, 0.f);
        if (a.beta) b = reinterpret_cast<const float4*>(a.beta)[i];
        v = make_float4(v.x * r * g.x + b.x, v.y * r * g.y + b.y, v.z * r * g.z + b.z, v.w * r * g.w + b.w);
        if constexpr (F32) *reinterpret_cast<float4*>(static_cast<float*>(a.xn) + base + 4 * i) = v;
        else *reinterpret_cast<uint2*>(static_cast<uint16_t*>(a.xn) + base + 4 * i) =
                 make_uint2((uint32_t)f_bf16(v.x) | ((uint32_t)f_bf16(v.y) << 16), (uint32_t)f_bf16(v.z) | ((uint32_t)f_bf16(v.w) << 16));
    };
#pragma unroll
    for (int k = 0; k < NS; ++k) {
        const int i = threadIdx.x + 256 * k;
        if (i < n4) emit(i, uv[k]);
    }
    for (int i = threadIdx.x + 256 * NS; i < n4; i += 256) emit(i, centred(i, again(i), mean));
}

constexpr int MAX_STREAMS = 16;
static int stream_rows(const StreamRows& a, int rows, bool f32, hipStream_t s) {
    if (a.streams <= 4) {
        if (f32) hipLaunchKernelGGL((stream_norm_rows_kernel<true, 4>), dim3(rows), dim3(256), 0, s, a);
        else hipLaunchKernelGGL((stream_norm_rows_kernel<false, 4>), dim3(rows), dim3(256), 0, s, a);
    } else {
        if (f32) hipLaunchKernelGGL((stream_norm_rows_kernel<true, MAX_STREAMS>), dim3(rows), dim3(256), 0, s, a);
        else hipLaunchKernelGGL((stream_norm_rows_kernel<false, MAX_STREAMS>), dim3(rows), dim3(256), 0, s, a);
    }
    return launch_status();
}

struct SideRows {
    const float* g;     // [slabs][rows][ld] partial sums of W_gate x
    int slabs;
    int64_t slab, ld;
    const uint16_t* table;
    int64_t table_ld;
    int offset, dim;
    const int* tokens;
    void* out;          // [rows][ld]
};
// grid rows: out = gelu_tanh(g) * e, e the token's row of the side table from column `offset`
template <bool F32>
__global__ __launch_bounds__(256) void side_rows_kernel(const SideRows a) {
    const uint16_t* e = a.table + (int64_t)a.tokens[blockIdx.x] * a.table_ld + a.offset;
    const int64_t base = blockIdx.x * a.ld;
    for (int i = threadIdx.x; i < a.dim; i += 256) {
        float v = 0.0f;
#pragma unroll 4
        for (int z = 0; z < a.slabs; ++z) v += a.g[base + z * a.slab + i];
        put_elem<F32>(a.out, base + i, gelu_tanh(v) * bf16_f(e[i]));
    }
}

struct MixRows {
    const float* raw;   // [rows][ld] projections
    int64_t ld;
    int heads, kv_heads, dim, vdim, rot_dim, rot_dims, kv_rank;
    const float *q_norm, *k_norm, *rope;
    float eps;
    int64_t pos0;
    const int64_t* d_past;  // position of row 0 instead of pos0, if given
    void* q;            // [rows][q_row]
    int64_t q_row;
    void *k, *v;        // caches
    int64_t k_row, v_row;
    int head_norm, values_are_keys;
};

// Elements c, c + 1 (c even) of a head of n values that starts at p, scaled by r and the norm weights w (NULL: none), rotated
// if c < rot_dims; zero past n.
__device__ __forceinline__ float2 rotated2(const float* p, const float* w, float r, int c, int n, int rot_dims, const float* cs) {
    float2 v = make_float2(0.0f, 0.0f);
    if (c >= n) return v;
    v.x = w ? p[c] * r * w[c] : p[c];
    if (c + 1 >= n) return v;
    v.y = w ? p[c + 1] * r * w[c + 1] : p[c + 1];
    if (c < rot_dims) {
        const float2 t = *reinterpret_cast<const float2*>(cs + c);
        v = make_float2(v.x * t.x - v.y * t.y, v.y * t.x + v.x * t.y);
    }
    return v;
}
template <bool F32>
__device__ __forceinline__ void put2(void* p, int64_t i, float2 v) {
    if constexpr (F32) *reinterpret_cast<float2*>(static_cast<float*>(p) + i) = v;
    else *reinterpret_cast<uint32_t*>(static_cast<uint16_t*>(p) + i) = (uint32_t)f_bf16(v.x) | ((uint32_t)f_bf16(v.y) << 16);
}
__device__ __forceinline__ float sumsq256(const float* p, int n) {  // this thread's share
    float s = 0.0f;
    if (((n | (int)(reinterpret_cast<uintptr_t>(p) >> 2)) & 3) == 0) {
#pragma unroll 4
        for (int i = threadIdx.x; i < n / 4; i += 256) {
            const float4 v = reinterpret_cast<const float4*>(p)[i];
            s = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, s))));
        }
    } else {
        for (int i = threadIdx.x; i < n; i += 256) s = fmaf(p[i], p[i], s);
    }
    return s;
}

// grid rows, dynamic LDS heads + kv_heads floats: q and k normed (over the whole projection, or per head) and rotated, k and v
// appended; heads padded to multiples of 8 with zeros
template <bool F32, bool Q32>
__global__ __launch_bounds__(256) void attention_prep_rows_kernel(const MixRows a) {
    __shared__ float red[4];
    extern __shared__ float s_r[];  // per head: one over the root mean square
    const int tid = threadIdx.x;
    const int64_t pos = (a.d_past ? *a.d_past : a.pos0) + blockIdx.x;
    const float *q = a.raw + blockIdx.x * a.ld, *k = q + a.heads * a.dim, *v = a.values_are_keys ? k : k + a.kv_heads * a.dim;
    const float* cs = a.rope + pos * a.rot_dims;
    const int nq = a.heads * a.dim, nk = a.kv_heads * a.dim, d8 = (a.dim + 7) & ~7, v8 = (a.vdim + 7) & ~7;
    float rq = 0.0f, rk = 0.0f;
    if (a.head_norm) {
        for (int h = tid >> 4; h < a.heads + a.kv_heads; h += 16) {  // 16 lanes per head
            float ss = 0.0f;
            for (int c = tid & 15; c < a.dim; c += 16) ss = fmaf(q[h * a.dim + c], q[h * a.dim + c], ss);
            ss = sum16(ss);
            if ((tid & 15) == 0) s_r[h] = 1.0f / sqrtf(ss / (float)a.dim + a.eps);
        }
        __syncthreads();
    } else {
        const float sq = sumsq256(q, nq), sk = sumsq256(k, nk);
        rq = 1.0f / sqrtf(block_sum<4>(sq, red) / (float)nq + a.eps);
        rk = 1.0f / sqrtf(block_sum<4>(sk, red) / (float)nk + a.eps);
    }
#pragma unroll 4
    for (int i = 2 * tid; i < a.heads * d8; i += 512) {
        const int h = i / d8, c = i % d8;
        put2<Q32>(a.q, blockIdx.x * a.q_row + i, rotated2(q + h * a.dim, a.q_norm + h * a.dim, a.head_norm ? s_r[h] : rq, c, a.dim, a.rot_dims, cs));
    }
#pragma unroll 2
    for (int i = 2 * tid; i < a.kv_heads * d8; i += 512) {
        const int h = i / d8, c = i % d8;
        put2<F32>(a.k, pos * a.k_row + i, rotated2(k + h * a.dim, a.k_norm + h * a.dim, a.head_norm ? s_r[a.heads + h] : rk, c, a.dim, a.rot_dims, cs));
    }
#pragma unroll 2
    for (int i = 2 * tid; i < a.kv_heads * v8; i += 512) {
        const int h = i / v8, c = i % v8;
        put2<F32>(a.v, pos * a.v_row + i, rotated2(v + h * a.vdim, nullptr, 1.0f, c, a.vdim, 0, nullptr));
    }
}
static size_t prep_lds(const MixRows& m) { return m.head_norm ? (size_t)(m.heads + m.kv_heads) * 4 : 0; }

// grid rows: latent normed and appended with the rotated key part; q per head [dim, 8-padded | rotated part, 8-padded]
template <bool F32>
__global__ __launch_bounds__(256) void latent_prep_rows_kernel(const MixRows a) {
    __shared__ float red[4];
    const int tid = threadIdx.x;
    const int64_t pos = a.pos0 + blockIdx.x;
    const int qd = a.dim + a.rot_dim, d8 = (a.dim + 7) & ~7, r8 = (a.rot_dim + 7) & ~7, rank8 = (a.kv_rank + 7) & ~7;
    const float *q = a.raw + blockIdx.x * a.ld, *c = q + a.heads * qd, *kr = c + a.kv_rank;
    const float* cs = a.rope + pos * a.rot_dims;
    const float r = 1.0f / sqrtf(block_sum<4>(sumsq256(c, a.kv_rank), red) / (float)a.kv_rank + a.eps);
    for (int i = 2 * tid; i < rank8 + r8; i += 512)
        put2<F32>(a.k, pos * a.k_row + i,
                  i < rank8 ? rotated2(c, a.k_norm, r, i, a.kv_rank, 0, nullptr) : rotated2(kr, nullptr, 1.0f, i - rank8, a.rot_dim, a.rot_dims, cs));
#pragma unroll 4
    for (int i = 2 * tid; i < a.heads * (d8 + r8); i += 512) {
        const int h = i / (d8 + r8), e = i % (d8 + r8);
        const float* qh = q + h * qd;
        put2<F32>(a.q, blockIdx.x * a.q_row + i,
                  e < d8 ? rotated2(qh, nullptr, 1.0f, e, a.dim, 0, nullptr) : rotated2(qh + a.dim, nullptr, 1.0f, e - d8, a.rot_dim, a.rot_dims, cs));
    }
}

// ---- the stack -----------------------------------------------------------------------------------
struct LayerRun {
    int block;
    int enters_pass;      // first block of a loop pass: its number, else -1
    void *k = nullptr, *v = nullptr;
    float *state = nullptr, *ring = nullptr;  // recurrent mixers: matrix state; token shift's or convolution's ring
};

struct BlockStack {
    ptm_block_config cfg{};
    std::vector<ptm_block> blocks;
    std::vector<const float*> rope;  // per block
    std::vector<LayerRun> runs;
    std::vector<void*> allocs;
    int wp = 0;           // padded width
    bool f32 = false;
    // token step
    float *emb = nullptr, *xa = nullptr, *xb = nullptr, *hb = nullptr, *proj = nullptr, *q = nullptr, *attn = nullptr,
          *act = nullptr, *gate = nullptr, *pO = nullptr, *pM = nullptr, *pL = nullptr;
    // what the last branch left: the residual, and the branch output that still has to be normed and added
    const float *x = nullptr, *pend_h = nullptr, *pend_w = nullptr;
    // prompt rows
    int rows = 0;
    void* slab = nullptr;
    int* r_tokens = nullptr;
    float *r_x = nullptr, *r_emb = nullptr, *r_h = nullptr, *r_proj = nullptr;
    void *r_xn = nullptr, *r_q = nullptr, *r_attn = nullptr, *r_act = nullptr, *r_gate = nullptr, *r_kv = nullptr;
    const float *r_pend_h = nullptr, *r_pend_w = nullptr;
    int r_slabs = 1;      // r_pend_h is the sum of that many slabs of a K-split product
    int64_t r_h_room = 0; // floats behind r_h
    // streams: blend weights per branch (stream_table), frequencies of the position sinusoid
    const float* blends = nullptr;
    const double* freq = nullptr;
    int branch = 0, r_branch = 0;  // the next branch's number
    const float *pend_store = nullptr, *r_pend_store = nullptr;
    float *r_hn = nullptr, *r_conv = nullptr, *r_scan = nullptr, *r_decay = nullptr;
    void *r_mix = nullptr, *r_low = nullptr;
    // all recurrent state, and its copy (blocks_state_copy)
    float *state = nullptr, *saved = nullptr;
    size_t state_floats = 0;
};

constexpr int64_t SPLIT_ROOM = (int64_t)8 << 20;  // floats for K-split partial sums beyond one set of rows

static int dev_alloc(BlockStack* b, size_t bytes, void** out) {
    int rc = hip_status(hipMalloc(out, bytes));
    if (rc != PTM_OK) return rc;
    b->allocs.push_back(*out);
    return hip_status(hipMemset(*out, 0, bytes));
}

static bool latent(const ptm_block& L) { return L.mixer == PTM_MIX_LATENT; }
static bool wkv(const ptm_block& L) { return L.mixer == PTM_MIX_WKV; }
static bool has_ssm(const ptm_block& L) { return L.ssm.heads > 0; }
static int ssm_channels(const ptm_ssm& m) { return m.heads * m.vdim + 2 * m.groups * m.state; }
// rows of `in`: what attention reads (wkv: everything), and all of them
static int attn_rows_of(const ptm_block& L) {
    if (wkv(L)) return 4 * L.wkv.heads * L.wkv.dim + L.wkv.rank;
    if (latent(L)) return L.heads * (L.dim + L.rot_dim) + L.kv_rank + L.rot_dim;
    return (L.heads + L.kv_heads) * L.dim + (L.values_are_keys ? 0 : L.kv_heads * L.vdim) + (L.out_gate ? L.heads * L.vdim : 0);
}
// prompt rows of a wkv mixer: floats between the r, k, v, g and w of a row
static int wkv_section(const ptm_block& L) { return up8(L.wkv.heads * L.wkv.dim); }
static int gate_row(const ptm_block& L) { return attn_rows_of(L) - L.heads * L.vdim; }
static int qkv_rows(const ptm_block& L) { return attn_rows_of(L) + (has_ssm(L) ? L.ssm.heads * (L.ssm.vdim + 1) + ssm_channels(L.ssm) : 0); }
// columns of `out`: attention's part, and all of them
static int attn_part(const ptm_block& L) { return wkv(L) ? L.wkv.heads * L.wkv.dim : L.heads * up8(L.vdim); }
static int attn_cols(const ptm_block& L) { return attn_part(L) + (has_ssm(L) ? L.ssm.heads * L.ssm.vdim : 0); }
static int up_rows(const ptm_block& L) { return L.ff_kind == PTM_FF_SWIGLU ? 2 * L.ff : L.ff; }
static int q_cols(const ptm_block& L) { return L.heads * (up8(L.dim) + (latent(L) ? up8(L.rot_dim) : 0)); }
static int64_t k_row(const ptm_block& L) { return latent(L) ? up8(L.kv_rank) + up8(L.rot_dim) : L.kv_heads * up8(L.dim); }
static int64_t v_row(const ptm_block& L) { return latent(L) ? 0 : L.kv_heads * up8(L.vdim); }
static int expand_rows(const ptm_block& L) { return L.heads * (up8(L.dim) + up8(L.vdim)); }

static int matrix_check(const ptm_qweight& w, int rows, int cols) {
    if (!w.data) return PTM_E_NULL;
    if (w.ggml_type != PTM_TYPE_BF16) return PTM_E_UNSUPPORTED;
    if (w.rows != rows || w.cols != cols || w.row_stride_bytes < 2 * (int64_t)up64(cols) || (w.row_stride_bytes & 15)) return PTM_E_SHAPE;
    if (!aligned16(w.data)) return PTM_E_ALIGN;
    return PTM_OK;
}

static int wkv_check(const ptm_block& L) {
    const ptm_wkv& m = L.wkv;
    if (m.heads <= 0 || m.dim <= 0 || m.rank <= 0 || (int64_t)m.heads * m.dim > 36864) return PTM_E_SHAPE;
    if (!recurrent_supported(m.dim) || m.rank > 8192 || has_ssm(L)) return PTM_E_UNSUPPORTED;
    if (!m.mu || !m.w0 || !m.u || !m.norm) return PTM_E_NULL;
    return matrix_check(m.w2, m.heads * m.dim, m.rank);
}
static int ssm_check(const ptm_ssm& m) {
    if (m.vdim <= 0 || m.state <= 0 || m.groups <= 0 || m.heads % m.groups || m.taps <= 0 || m.norm_groups <= 0 || m.heads > 36864 || m.vdim > 36864 ||
        (int64_t)m.heads * m.vdim > 36864 || (int64_t)m.heads * m.vdim % m.norm_groups)
        return PTM_E_SHAPE;
    if (!recurrent_supported(m.state) || m.norm_groups > 512 || m.taps > 4096 || (int64_t)m.groups * m.state > 36864) return PTM_E_UNSUPPORTED;
    return m.conv && m.conv_b && m.dt_bias && m.neg_a && m.D && m.norm ? PTM_OK : PTM_E_NULL;
}

static int block_check(const ptm_block& L, int hidden, int side_dim, int streams) {
    if (L.mixer != PTM_MIX_ATTENTION && L.mixer != PTM_MIX_LATENT && L.mixer != PTM_MIX_WKV) return PTM_E_UNSUPPORTED;
    if (L.ff_kind != PTM_FF_RELU2 && L.ff_kind != PTM_FF_SWIGLU) return PTM_E_UNSUPPORTED;
    if (streams > 0) {
        if (L.norm1b || L.norm2b || L.side_gate.data) return PTM_E_UNSUPPORTED;
        for (int q = 0; q < (L.ff > 0 ? 2 : 1); ++q)
            if (!L.hc_in[q] || !L.hc_out[q] || !L.hc_mix[q]) return PTM_E_NULL;
    } else if (L.norm1_bias || L.norm2_bias || wkv(L) || has_ssm(L)) {
        return PTM_E_UNSUPPORTED;  // the prologues of these live with the streams'
    }
    if ((L.values_are_keys || L.out_gate || L.sink || L.head_norm || L.out_scale != 0.0f) && L.mixer != PTM_MIX_ATTENTION) return PTM_E_UNSUPPORTED;
    if (latent(L) && has_ssm(L)) return PTM_E_UNSUPPORTED;
    if (L.ssm.heads < 0 || (L.values_are_keys && L.vdim != L.dim)) return PTM_E_SHAPE;
    if (wkv(L) || has_ssm(L)) {
        const int rc = wkv(L) ? wkv_check(L) : ssm_check(L.ssm);
        if (rc) return rc;
    }
    if (!wkv(L) && (L.heads <= 0 || L.dim <= 0 || L.vdim <= 0 || L.window < 0 || L.keep_first < 0 || L.softcap < 0.0f)) return PTM_E_SHAPE;
    if (L.rot.dims < 0 || (L.rot.dims & 1)) return PTM_E_SHAPE;
    int rc;
    if (wkv(L)) {
        if (hidden > 36864 || L.ff > 36864) return PTM_E_UNSUPPORTED;
    } else if (latent(L)) {
        if (L.rot_dim <= 0 || L.kv_rank <= 0 || L.rot.dims > L.rot_dim) return PTM_E_SHAPE;
        if (L.dim > 1024 || L.kv_rank > 2048 || L.kv_rank + L.rot_dim > 8000) return PTM_E_UNSUPPORTED;
        if (!L.k_norm) return PTM_E_NULL;
        if ((rc = matrix_check(L.expand, expand_rows(L), L.kv_rank))) return rc;
    } else {
        if (L.kv_heads <= 0 || L.heads % L.kv_heads || L.rot.dims > L.dim) return PTM_E_SHAPE;
        if (!L.q_norm || !L.k_norm) return PTM_E_NULL;
    }
    if (L.vdim > 2048 || L.dim > 4000 || attn_cols(L) > 36864 || hidden > 36864 || L.ff > 36864) return PTM_E_UNSUPPORTED;
    if (!L.norm1 || (streams <= 0 && !L.norm1b)) return PTM_E_NULL;
    if ((rc = matrix_check(L.in, qkv_rows(L), hidden)) || (rc = matrix_check(L.out, hidden, attn_cols(L)))) return rc;
    if (L.ff < 0) return PTM_E_SHAPE;
    if (L.ff > 0) {
        if (!L.norm2 || (streams <= 0 && !L.norm2b)) return PTM_E_NULL;
        if ((rc = matrix_check(L.up, up_rows(L), hidden)) || (rc = matrix_check(L.down, hidden, L.ff))) return rc;
    }
    if (L.side_gate.data) {
        if (side_dim <= 0 || L.side_offset < 0) return PTM_E_SHAPE;
        if (!L.side_norm) return PTM_E_NULL;
        if ((rc = matrix_check(L.side_gate, side_dim, hidden)) || (rc = matrix_check(L.side_proj, hidden, side_dim))) return rc;
    }
    return PTM_OK;
}

// attention of the block's decode step, without pointers into the caches when run is NULL
static ptm_attention_args decode_args(const BlockStack* b, const ptm_block& L, const LayerRun* run) {
    ptm_attention_args a{};
    const int es = b->f32 ? 4 : 2;
    a.rows = 1;
    a.heads = L.heads;
    a.window = L.window;
    a.keep_first = L.keep_first;
    a.scale = L.scale;
    a.softcap = L.softcap;
    a.fp32 = b->f32;
    a.Q = b->q;
    if (latent(L)) {
        a.kv_heads = 1;
        a.dim1 = a.vdim = up8(L.kv_rank);
        a.dim2 = up8(L.rot_dim);
        a.k1_row = a.k2_row = a.v_row = k_row(L);
        if (run) {
            a.K1 = a.V = run->k;
            a.K2 = static_cast<uint8_t*>(run->k) + (size_t)a.dim1 * es;
        }
    } else {
        a.kv_heads = L.kv_heads;
        a.dim1 = a.k1_head = up8(L.dim);
        a.vdim = a.v_head = up8(L.vdim);
        a.k1_row = k_row(L);
        a.v_row = v_row(L);
        if (run) { a.K1 = run->k; a.V = run->v; }
    }
    a.q_row = L.heads * (a.dim1 + a.dim2);
    a.o_row = L.heads * a.vdim;
    a.sink = L.sink;
    a.out_scale = L.out_scale;
    if (L.out_gate) {
        a.gate = b->proj ? b->proj + gate_row(L) : nullptr;
        a.gate_head = L.vdim;
    }
    return a;
}

// state and ring of every run with a recurrent mixer, in one piece, and as much again for a copy
static int alloc_states(BlockStack* b) {
    auto sizes = [&](const ptm_block& L, size_t* state, size_t* ring) {
        *state = *ring = 0;
        if (wkv(L)) {
            *state = (size_t)recurrent_state_floats(L.wkv.heads, L.wkv.dim, L.wkv.dim);
            *ring = 2 * (size_t)b->wp;
        } else if (has_ssm(L)) {
            *state = (size_t)recurrent_state_floats(L.ssm.heads, L.ssm.state, L.ssm.vdim);
            *ring = ((size_t)L.ssm.taps * (size_t)ssm_channels(L.ssm) + 63) & ~(size_t)63;
        }
    };
    size_t total = 0, st, ring;
    for (const LayerRun& r : b->runs) {
        sizes(b->blocks[(size_t)r.block], &st, &ring);
        total += st + ring;
    }
    b->state_floats = total;
    if (!total) return PTM_OK;
    int rc = dev_alloc(b, total * 4, reinterpret_cast<void**>(&b->state));
    if (rc == PTM_OK) rc = dev_alloc(b, total * 4, reinterpret_cast<void**>(&b->saved));
    if (rc != PTM_OK) return rc;
    float* p = b->state;
    for (LayerRun& r : b->runs) {
        sizes(b->blocks[(size_t)r.block], &st, &ring);
        if (!st) continue;
        r.state = p;
        r.ring = p + st;
        p += st + ring;
    }
    return PTM_OK;
}

// Blend weights, S = streams.  Branch e (a run's mixer or feed-forward, in order; the head is one more): what its output does to the
// streams [S][S + 1]; the vector it reads, from the streams as they are [S + 1]; and from the streams before the branch ahead
// and that branch's output [S + 1].
static size_t stream_branch_floats(int S) { return (size_t)(S + 2) * (size_t)(S + 1); }
static const float* branch_store(const BlockStack* b, int e) { return b->blends + stream_branch_floats(b->cfg.streams) * (size_t)e; }
static const float* branch_blend(const BlockStack* b, int e, bool pending) {
    const int S = b->cfg.streams;
    return branch_store(b, e) + (size_t)(S + (pending ? 1 : 0)) * (size_t)(S + 1);
}
static int stream_tables(BlockStack* b) {
    const ptm_block_config& c = b->cfg;
    const int S = c.streams;
    std::vector<float> t;
    std::vector<double> prev;  // the branch ahead, [S][S + 1]
    auto branch = [&](const float* in, const float* out, const float* mix) {
        const size_t base = t.size();
        t.resize(base + stream_branch_floats(S), 0.0f);
        float *store = t.data() + base, *plain = store + S * (S + 1), *pending = plain + S + 1;
        for (int i = 0; i < S; ++i) plain[i] = in ? in[i] : 1.0f;
        if (!prev.empty())
            for (int k = 0; k <= S; ++k) {
                double v = 0.0;
                for (int i = 0; i < S; ++i) v += (double)plain[i] * prev[(size_t)(i * (S + 1) + k)];
                pending[k] = (float)v;
            }
        if (!in) return;
        for (int i = 0; i < S; ++i) {
            for (int k = 0; k < S; ++k) store[i * (S + 1) + k] = mix[k * S + i];
            store[i * (S + 1) + S] = out[i];
        }
        prev.assign(store, store + S * (S + 1));
    };
    for (const LayerRun& r : b->runs) {
        const ptm_block& L = b->blocks[(size_t)r.block];
        for (int q = 0; q < (L.ff > 0 ? 2 : 1); ++q) branch(L.hc_in[q], L.hc_out[q], L.hc_mix[q]);
    }
    branch(nullptr, nullptr, nullptr);
    void* d = nullptr;
    int rc = dev_alloc(b, t.size() * 4, &d);
    if (rc == PTM_OK) rc = hip_status(hipMemcpy(d, t.data(), t.size() * 4, hipMemcpyHostToDevice));
    b->blends = static_cast<const float*>(d);
    if (rc == PTM_OK && c.position_base > 0.0) {
        std::vector<double> f((size_t)b->wp / 2 + 1, 0.0);
        for (int i = 0; 2 * i < c.hidden; ++i) f[(size_t)i] = std::pow(c.position_base, -2.0 * i / c.hidden);
        rc = dev_alloc(b, f.size() * 8, &d);
        if (rc == PTM_OK) rc = hip_status(hipMemcpy(d, f.data(), f.size() * 8, hipMemcpyHostToDevice));
        b->freq = static_cast<const double*>(d);
    }
    return rc;
}

int blocks_create(const ptm_block_config& c, BlockStack** out) {
    *out = nullptr;
    if (!c.blocks || !c.out_norm) return PTM_E_NULL;
    if (c.vocab <= 0 || c.hidden <= 0 || c.n_blocks <= 0 || c.max_seq <= 0) return PTM_E_SHAPE;
    if (c.precision != PTM_PRECISION_16 && c.precision != PTM_PRECISION_32) return PTM_E_UNSUPPORTED;
    if (c.loop_times < 0 || (c.loop_times > 0 && (c.loop_start < 0 || c.loop_start >= c.loop_stop || c.loop_stop > c.n_blocks))) return PTM_E_SHAPE;
    if (c.loop_times > 0 && !c.loop_step) return PTM_E_NULL;
    if (c.streams < 0 || c.position_base < 0.0) return PTM_E_SHAPE;
    if (c.streams > MAX_STREAMS) return PTM_E_UNSUPPORTED;
    if (c.streams > 0 ? c.loop_times > 0 || c.side_table.data : c.position_base > 0.0 || c.out_norm_bias) return PTM_E_UNSUPPORTED;
    int rc;
    if ((rc = matrix_check(c.lm_head, c.vocab, c.hidden)) || (rc = matrix_check(c.embedding, c.vocab, c.hidden))) return rc;
    if (c.side_table.data && ((rc = matrix_check(c.side_table, c.vocab, c.side_table.cols)))) return rc;
    for (int i = 0; i < c.n_blocks; ++i) {
        if ((rc = block_check(c.blocks[i], c.hidden, c.side_dim, c.streams))) return rc;
        if (c.blocks[i].side_gate.data && (!c.side_table.data || c.blocks[i].side_offset + c.side_dim > c.side_table.cols)) return PTM_E_SHAPE;
    }
    BlockStack* b = new (std::nothrow) BlockStack();
    if (!b) return PTM_E_STATE;
    b->cfg = c;
    b->blocks.assign(c.blocks, c.blocks + c.n_blocks);
    b->cfg.blocks = b->blocks.data();
    b->wp = up64(c.hidden);
    b->f32 = c.precision == PTM_PRECISION_32;
    for (int i = 0; i < c.n_blocks; ++i) {
        if (c.loop_times > 0 && i == c.loop_start) {
            for (int t = 0; t < c.loop_times; ++t)
                for (int k = c.loop_start; k < c.loop_stop; ++k) b->runs.push_back({k, k == c.loop_start ? t : -1});
            i = c.loop_stop - 1;
        } else {
            b->runs.push_back({i, -1});
        }
    }
    const int es = b->f32 ? 4 : 2;
    size_t proj = 0, q = 0, attn = 0, act = 64, pO = 0, pM = 0;
    rc = PTM_OK;
    for (int i = 0; rc == PTM_OK && i < c.n_blocks; ++i) {
        const ptm_block& L = b->blocks[(size_t)i];
        auto grow = [](size_t& v, size_t n) { v = v > n ? v : n; };
        grow(proj, (size_t)up64(qkv_rows(L)));
        grow(attn, (size_t)up64(attn_cols(L)));
        grow(act, (size_t)up64(L.ff));
        if (wkv(L)) {
            b->rope.push_back(nullptr);
            continue;
        }
        const ptm_attention_args a = decode_args(b, L, nullptr);
        const size_t splits = (size_t)decode_attention_splits(a, c.max_seq);
        grow(q, (size_t)a.q_row);
        grow(pO, splits * (size_t)a.o_row);
        grow(pM, splits * (size_t)L.heads);
        // rotation table, shared with an earlier block that rotates alike
        const float* table = nullptr;
        for (int k = 0; k < i && !table; ++k) {
            const ptm_rotation &r = b->blocks[(size_t)k].rot, &n = L.rot;
            if (!wkv(b->blocks[(size_t)k]) && r.dims == n.dims && r.base == n.base && r.factor == n.factor && r.original == n.original && r.fast == n.fast && r.slow == n.slow)
                table = b->rope[(size_t)k];
        }
        if (!table) {
            std::vector<float> host((size_t)c.max_seq * (size_t)(L.rot.dims > 0 ? L.rot.dims : 2), 0.0f);
            if (L.rot.dims > 0) rc = ptm_rope_pairs_host(host.data(), c.max_seq, &L.rot);
            void* dev = nullptr;
            if (rc == PTM_OK) rc = dev_alloc(b, host.size() * 4, &dev);
            if (rc == PTM_OK) rc = hip_status(hipMemcpy(dev, host.data(), host.size() * 4, hipMemcpyHostToDevice));
            table = static_cast<const float*>(dev);
        }
        b->rope.push_back(table);
    }
    for (size_t i = 0; rc == PTM_OK && i < b->runs.size(); ++i) {
        const ptm_block& L = b->blocks[(size_t)b->runs[i].block];
        if (wkv(L)) continue;
        // 64 values behind the last row: a GEMM over latents reads whole steps of 64 columns
        rc = dev_alloc(b, ((size_t)c.max_seq * (size_t)k_row(L) + 64) * es, &b->runs[i].k);
        if (rc == PTM_OK && !latent(L)) rc = dev_alloc(b, ((size_t)c.max_seq * (size_t)v_row(L) + 64) * es, &b->runs[i].v);
    }
    if (rc == PTM_OK) rc = alloc_states(b);
    if (rc == PTM_OK && c.streams > 0) rc = stream_tables(b);
    const size_t S = (size_t)(c.streams > 0 ? c.streams : 1);
    auto vec = [&](float*& p, size_t n) { if (rc == PTM_OK) rc = dev_alloc(b, (n + 64) * 4, reinterpret_cast<void**>(&p)); };
    vec(b->emb, S * (size_t)b->wp);
    vec(b->xa, S * (size_t)b->wp);
    vec(b->xb, S * (size_t)b->wp);
    vec(b->hb, (size_t)b->wp);
    vec(b->proj, proj);
    vec(b->q, q);
    vec(b->attn, attn > q ? attn : q);
    vec(b->act, act);
    vec(b->gate, (size_t)up64(c.side_dim > 0 ? c.side_dim : 1));
    vec(b->pO, pO);
    vec(b->pM, pM);
    vec(b->pL, pM);
    // the clears above run on the null stream, which the decoder's own stream does not wait for
    if (rc == PTM_OK) rc = hip_status(hipStreamSynchronize(nullptr));
    if (rc != PTM_OK) { blocks_destroy(b); return rc; }
    dense_gemv_init();
    *out = b;
    return PTM_OK;
}

void blocks_destroy(BlockStack* b) {
    if (!b) return;
    for (void* p : b->allocs) (void)hipFree(p);
    if (b->slab) (void)hipFree(b->slab);
    delete b;
}

int blocks_runs(const BlockStack* b) { return (int)b->runs.size(); }
bool blocks_recurrent(const BlockStack* b) { return b->state_floats > 0; }
int blocks_state_copy(BlockStack* b, bool restore, hipStream_t s) {
    if (!b->state_floats) return PTM_OK;
    return hip_status(hipMemcpyAsync(restore ? b->state : b->saved, restore ? b->saved : b->state, b->state_floats * 4, hipMemcpyDeviceToDevice, s));
}

#define PTM_TRY(call) do { rc = (call); if (rc != PTM_OK) return rc; } while (0)

static MixRows mix_rows(const BlockStack* b, const ptm_block& L, int block, const LayerRun& run) {
    MixRows m{};
    m.heads = L.heads;
    m.kv_heads = L.kv_heads;
    m.dim = L.dim;
    m.vdim = L.vdim;
    m.rot_dim = L.rot_dim;
    m.rot_dims = L.rot.dims;
    m.kv_rank = L.kv_rank;
    m.q_norm = L.q_norm;
    m.k_norm = L.k_norm;
    m.rope = b->rope[(size_t)block];
    m.eps = b->cfg.eps;
    m.k = run.k;
    m.v = run.v;
    m.k_row = k_row(L);
    m.v_row = v_row(L);
    m.head_norm = L.head_norm;
    m.values_are_keys = L.values_are_keys;
    return m;
}

static SsmShape ssm_shape(const ptm_ssm& m) {
    return {m.heads, m.vdim, m.state, m.groups, m.taps, m.norm_groups, m.conv, m.conv_b, m.dt_bias, m.neg_a, m.D, m.norm, m.scale != 0.0f ? m.scale : 1.0f};
}

static int trace_rows(const BlockStack* b, const float* x, int64_t stride, int rows, float* out, hipStream_t s) {
    hipLaunchKernelGGL(copy_rows_kernel, dim3(rows), dim3(256), 0, s, x, b->cfg.streams, stride, b->wp, b->cfg.hidden, out);
    return launch_status();
}

static int add_pending(BlockStack* b, hipStream_t s) {  // in place, for traced steps
    if (!b->pend_h) return PTM_OK;
    if (b->cfg.streams > 0) {
        const StreamRows r{const_cast<float*>(b->x), b->cfg.streams, b->wp, b->pend_h, 1, 0, b->pend_store, nullptr, nullptr, nullptr, nullptr,
                           b->cfg.hidden, b->wp, b->cfg.eps};
        b->pend_h = nullptr;
        return stream_rows(r, 1, true, s);
    }
    if (b->x == b->emb) {  // a loop adds the embedding output again: it stays as it is
        const int rc = ptm_copy(b->emb, b->xa, b->wp, s);
        if (rc != PTM_OK) return rc;
        b->x = b->xa;
    }
    hipLaunchKernelGGL(residual_norm_rows_kernel<true>, dim3(1), dim3(256), 0, s, const_cast<float*>(b->x), b->pend_h, 1, (int64_t)0, b->pend_w,
                       (const float*)nullptr, (const float*)nullptr, (const float*)nullptr, (void*)nullptr, b->cfg.hidden, b->wp, b->cfg.eps);
    b->pend_h = b->pend_w = nullptr;
    return launch_status();
}

// one token's attention from b->proj to the front of b->attn
static int attention_step(BlockStack* b, const ptm_block& L, const LayerRun& run, const int64_t* d_past, hipStream_t s) {
    int rc;
    DecodeAttention d{};
    d.a = decode_args(b, L, &run);
    d.d_past = d_past;
    d.max_seq = b->cfg.max_seq;
    d.pO = b->pO;
    d.pM = b->pM;
    d.pL = b->pL;
    const bool tiled = decode_attention_tiled(d.a);
    const int splits = decode_attention_splits(d.a, b->cfg.max_seq);
    if (latent(L)) {
        const LatentStep ls{b->proj, L.k_norm, b->rope[(size_t)run.block], static_cast<const uint16_t*>(L.expand.data),
                            L.expand.row_stride_bytes / 2, L.heads, L.dim, L.rot_dim, L.rot.dims, L.kv_rank, L.vdim, b->cfg.eps, d_past,
                            b->q, tiled, run.k, b->f32};
        PTM_TRY(latent_absorb(ls, s));
        if (tiled) {
            PTM_TRY(decode_attention(d, s));
            PTM_TRY(latent_out(ls, b->pO, b->pM, b->pL, splits, d.a.vdim, b->attn, s));
        } else {
            d.a.O = b->pO;
            PTM_TRY(attention_rows(d.a, d_past, true, s));
            PTM_TRY(latent_out(ls, b->pO, nullptr, nullptr, 1, d.a.vdim, b->attn, s));
        }
    } else if (tiled) {
        d.raw = b->proj;
        d.q_norm = L.q_norm;
        d.k_norm = L.k_norm;
        d.rope = b->rope[(size_t)run.block];
        d.dim = L.dim;
        d.vdim_true = L.vdim;
        d.rot_dims = L.rot.dims;
        d.eps = b->cfg.eps;
        d.head_norm = L.head_norm;
        d.values_are_keys = L.values_are_keys;
        d.k_cache = run.k;
        d.v_cache = run.v;
        PTM_TRY(decode_attention(d, s));
        PTM_TRY(decode_attention_merge(b->pO, b->pM, b->pL, splits, d.a, b->attn, s));
    } else {
        MixRows m = mix_rows(b, L, run.block, run);
        m.raw = b->proj;
        m.d_past = d_past;
        m.q = b->q;
        m.q_row = d.a.q_row;
        if (b->f32) hipLaunchKernelGGL((attention_prep_rows_kernel<true, true>), dim3(1), dim3(256), prep_lds(m), s, m);
        else hipLaunchKernelGGL((attention_prep_rows_kernel<false, true>), dim3(1), dim3(256), prep_lds(m), s, m);
        PTM_TRY(launch_status());
        d.a.O = b->attn;
        PTM_TRY(attention_rows(d.a, d_past, true, s));
    }
    return PTM_OK;
}

// prologue of a projection in front of branch b->branch: takes in whatever is pending; the new streams go to the other buffer
static void take_streams(BlockStack* b, DenseGemv& g) {
    g.streams = b->cfg.streams;
    g.eps = b->cfg.eps;
    g.x = b->x;
    g.x_stride = b->wp;
    g.blend = branch_blend(b, b->branch, b->pend_h != nullptr);
    if (b->pend_h) {
        g.h = b->pend_h;
        g.store = b->pend_store;
        g.xout = b->x == b->xa ? b->xb : b->xa;
        b->x = g.xout;
    }
    b->pend_h = b->pend_w = b->pend_store = nullptr;
}

int blocks_token(BlockStack* b, const int* d_token, const int64_t* d_past, float* trace, hipStream_t s) {
    const ptm_block_config& c = b->cfg;
    int rc;
    if (c.streams > 0)
        hipLaunchKernelGGL(embed_streams_kernel, dim3(1, (b->wp + 511) / 512), dim3(128), 0, s, static_cast<const uint16_t*>(c.embedding.data),
                           c.embedding.row_stride_bytes / 2, d_token, b->freq, d_past, (int64_t)0, c.hidden, b->wp, c.streams, (int64_t)b->wp, b->emb);
    else
        hipLaunchKernelGGL(embed_bf16_rows_kernel, dim3(1, (b->wp + 511) / 512), dim3(128), 0, s, static_cast<const uint16_t*>(c.embedding.data),
                           c.embedding.row_stride_bytes / 2, d_token, b->wp, b->emb, (float*)nullptr);
    PTM_TRY(launch_status());
    b->x = b->emb;
    b->pend_h = b->pend_w = b->pend_store = nullptr;
    b->branch = 0;
    const float *add0 = nullptr, *add1 = nullptr;
    auto weight = [](DenseGemv& g, const ptm_qweight& w, float* y) {
        g.W = static_cast<const uint16_t*>(w.data);
        g.ld = w.row_stride_bytes / 2;
        g.N = w.rows;
        g.K = w.cols;
        g.y = y;
    };
    // a projection of the residual: takes in whatever is pending and leaves the sum in the other residual buffer
    auto from_x = [&](DenseGemv& g) {
        if (c.streams > 0) {
            take_streams(b, g);
            return dense_gemv(g, s);
        }
        g.x = b->x;
        g.eps = c.eps;
        g.h = b->pend_h;
        g.hw = b->pend_w;
        g.add0 = add0;
        g.add1 = add1;
        if (g.h || add0 || add1) {
            g.xout = b->x == b->xa ? b->xb : b->xa;
            b->x = g.xout;
        }
        b->pend_h = b->pend_w = add0 = add1 = nullptr;
        return dense_gemv(g, s);
    };
    auto branch_out = [&](const ptm_qweight& w, const float* x, const float* post, const ptm_ssm* ssm = nullptr) {
        DenseGemv g;
        weight(g, w, b->hb);
        g.x = x;
        if (ssm && ssm->heads > 0) {
            g.tail_n = ssm->heads * ssm->vdim;
            g.tail0 = w.cols - g.tail_n;
            g.tail_parts = ssm->norm_groups;
            g.tail_norm = ssm->norm;
            g.tail_scale = ssm->scale != 0.0f ? ssm->scale : 1.0f;
            g.eps = c.eps;
        }
        b->pend_h = b->hb;
        b->pend_w = post;
        if (c.streams > 0) b->pend_store = branch_store(b, b->branch++);
        return dense_gemv(g, s);
    };
    for (size_t ri = 0; ri < b->runs.size(); ++ri) {
        const LayerRun& run = b->runs[ri];
        const ptm_block& L = b->blocks[(size_t)run.block];
        if (run.enters_pass >= 0) {
            add0 = run.enters_pass > 0 ? b->emb : nullptr;
            add1 = c.loop_step + (int64_t)run.enters_pass * b->wp;
        }
        {
            DenseGemv g;
            weight(g, L.in, b->proj);
            g.gamma = L.norm1;
            g.beta = L.norm1_bias;
            if (wkv(L)) {
                const int hd = L.wkv.heads * L.wkv.dim;
                g.mu = L.wkv.mu;
                g.shift = run.ring;
                g.d_past = d_past;
                g.sections = 5;
                for (int i = 0; i < 5; ++i) g.section_row[i] = i * hd;
                g.section_row[5] = g.N;
            }
            PTM_TRY(from_x(g));
        }
        if (wkv(L)) {
            const ptm_wkv& m = L.wkv;
            PTM_TRY(wkv_step({b->proj, static_cast<const uint16_t*>(m.w2.data), m.w2.row_stride_bytes / 2, m.heads, m.dim, m.rank, m.w0, m.u, m.norm,
                              c.eps, d_past, run.state, b->attn}, s));
        } else {
            PTM_TRY(attention_step(b, L, run, d_past, s));
            if (has_ssm(L)) PTM_TRY(ssm_step({ssm_shape(L.ssm), b->proj + attn_rows_of(L), d_past, run.ring, run.state, b->attn + attn_part(L)}, s));
        }
        PTM_TRY(branch_out(L.out, b->attn, L.norm1b, &L.ssm));
        if (trace) {
            PTM_TRY(add_pending(b, s));
            PTM_TRY(trace_rows(b, b->x, b->wp, 1, trace + (2 * ri) * (size_t)c.hidden, s));
        }
        if (L.ff > 0) {
            DenseGemv g;
            weight(g, L.up, b->act);
            g.N = L.ff;
            g.gamma = L.norm2;
            g.beta = L.norm2_bias;
            g.epilogue = L.ff_kind == PTM_FF_SWIGLU ? GEMV_SWIGLU : GEMV_RELU2;
            PTM_TRY(from_x(g));
            PTM_TRY(branch_out(L.down, b->act, L.norm2b));
        }
        if (L.side_gate.data) {
            DenseGemv g;
            weight(g, L.side_gate, b->gate);
            g.epilogue = GEMV_SIDE;
            g.side = static_cast<const uint16_t*>(c.side_table.data);
            g.side_ld = c.side_table.row_stride_bytes / 2;
            g.side_off = L.side_offset;
            g.d_token = d_token;
            PTM_TRY(from_x(g));
            PTM_TRY(branch_out(L.side_proj, b->gate, L.side_norm));
        }
        if (trace) {
            PTM_TRY(add_pending(b, s));
            PTM_TRY(trace_rows(b, b->x, b->wp, 1, trace + (2 * ri + 1) * (size_t)c.hidden, s));
        }
    }
    return PTM_OK;
}

int blocks_head(BlockStack* b, int row, float* logits, float* xn, int64_t* d_next, void* argmax_ws, const ArgmaxAdvance* adv,
                hipStream_t s) {
    const ptm_block_config& c = b->cfg;
    DenseGemv g;
    g.W = static_cast<const uint16_t*>(c.lm_head.data);
    g.ld = c.lm_head.row_stride_bytes / 2;
    g.N = c.vocab;
    g.K = c.hidden;
    g.x = row < 0 ? b->x : b->r_x + (int64_t)row * b->wp;
    g.h = row < 0 ? b->pend_h : b->r_pend_h ? b->r_pend_h + (int64_t)row * b->wp : nullptr;
    g.hw = row < 0 ? b->pend_w : b->r_pend_w;
    if (c.streams > 0) {  // nothing reads the streams after this: they are not stored
        g.streams = c.streams;
        g.x_stride = row < 0 ? b->wp : (int64_t)b->rows * b->wp;
        g.blend = branch_blend(b, row < 0 ? b->branch : b->r_branch, g.h != nullptr);
        g.hw = nullptr;
        g.beta = c.out_norm_bias;
    }
    g.out_scale = c.logit_scale != 0.0f ? c.logit_scale : 1.0f;
    g.gamma = c.out_norm;
    g.eps = c.eps;
    g.xn_out = xn;
    g.y = logits;
    if (!adv) return dense_gemv(g, s);
    const int wgs = dense_gemv_workgroups(g);
    g.epilogue = GEMV_ARGMAX;
    g.part_val = static_cast<float*>(argmax_ws);
    g.part_idx = reinterpret_cast<int*>(g.part_val + wgs);
    const int rc = dense_gemv(g, s);
    return rc != PTM_OK ? rc : argmax_finish(g.part_val, g.part_idx, wgs, d_next, *adv, s);
}

// ---- prompt rows -----------------------------------------------------------------------------------
// first position whose latents a chunk at pos0 expands, and how many positions a chunk of `rows` rows may expand at most
static int64_t expand_from(const ptm_block& L, int64_t pos0) {
    return L.window > 0 && !L.keep_first && pos0 - L.window + 1 > 0 ? pos0 - L.window + 1 : 0;
}
static size_t expand_positions(const BlockStack* b, const ptm_block& L, int rows) {
    const size_t all = (size_t)b->cfg.max_seq, n = (size_t)rows + (size_t)L.window;
    return L.window > 0 && !L.keep_first && n < all ? n : all;
}

int blocks_reserve(BlockStack* b, int rows) {
    if (b->rows >= rows) return PTM_OK;
    if (b->slab) { (void)hipFree(b->slab); b->slab = nullptr; b->rows = 0; }
    const ptm_block_config& c = b->cfg;
    const size_t R = (size_t)rows, es = b->f32 ? 4 : 2, W = (size_t)b->wp;
    const size_t S = (size_t)(c.streams > 0 ? c.streams : 1);
    size_t proj = 0, q = 0, attn = 0, act = 64, kv = 0, shifted = 0, low = 0, conv = 0, scan = 0, steps = 0;
    for (const ptm_block& L : b->blocks) {
        auto grow = [](size_t& v, size_t n) { v = v > n ? v : n; };
        grow(proj, (size_t)(wkv(L) ? 5 * wkv_section(L) : up64(qkv_rows(L))));
        if (wkv(L)) {
            shifted = R * W;
            grow(low, (size_t)up64(L.wkv.rank));
            grow(scan, (size_t)scan_slabs(L.wkv.dim) * (size_t)(L.wkv.heads * L.wkv.dim));
        } else {
            grow(q, (size_t)q_cols(L));
        }
        if (has_ssm(L)) {
            grow(conv, (size_t)ssm_channels(L.ssm));
            grow(scan, (size_t)scan_slabs(L.ssm.state) * (size_t)(L.ssm.heads * L.ssm.vdim));
            grow(steps, 2 * (size_t)L.ssm.heads);
        }
        grow(attn, (size_t)up64(attn_cols(L)));
        grow(act, (size_t)up64(L.ff));
        if (latent(L)) grow(kv, expand_positions(b, L, rows) * (size_t)expand_rows(L));
    }
    const size_t wide = W > low ? W : low;  // r_h also takes the decay's low-rank products
    size_t off = 0;
    auto take = [&](size_t bytes) { const size_t o = off; off += (bytes + 511) & ~(size_t)255; return o; };
    const size_t o_tok = take(4 * R), o_x = take(4 * S * R * W), o_e = take(4 * R * W), o_h = take(4 * (R * wide + (size_t)SPLIT_ROOM)), o_p = take(4 * R * proj),
                 o_xn = take(es * R * W), o_q = take(es * R * q), o_at = take(es * R * attn), o_ac = take(es * R * act),
                 o_g = take(es * R * (size_t)up64(c.side_dim > 0 ? c.side_dim : 1)), o_kv = take(es * kv),
                 o_hn = take(4 * shifted), o_mix = take(es * 5 * shifted), o_low = take(es * R * low), o_cv = take(4 * R * conv), o_sc = take(4 * R * scan),
                 o_st = take(4 * R * steps);
    int rc = hip_status(hipMalloc(&b->slab, off));
    if (rc != PTM_OK) return rc;
    if ((rc = hip_status(hipMemset(b->slab, 0, off))) != PTM_OK) return rc;
    if ((rc = hip_status(hipStreamSynchronize(nullptr))) != PTM_OK) return rc;  // before the decoder's stream writes there
    uint8_t* p = static_cast<uint8_t*>(b->slab);
    b->r_tokens = (int*)(p + o_tok);
    b->r_x = (float*)(p + o_x);
    b->r_emb = (float*)(p + o_e);
    b->r_h = (float*)(p + o_h);
    b->r_proj = (float*)(p + o_p);
    b->r_h_room = (int64_t)(R * wide) + SPLIT_ROOM;
    b->r_xn = p + o_xn;
    b->r_q = p + o_q;
    b->r_attn = p + o_at;
    b->r_act = p + o_ac;
    b->r_gate = p + o_g;
    b->r_kv = p + o_kv;
    b->r_hn = (float*)(p + o_hn);
    b->r_mix = p + o_mix;
    b->r_low = p + o_low;
    b->r_conv = (float*)(p + o_cv);
    b->r_scan = (float*)(p + o_sc);
    b->r_decay = (float*)(p + o_st);
    b->rows = rows;
    return PTM_OK;
}

static DenseGemm product(const BlockStack* b, const ptm_qweight& w, const void* A, int64_t lda, int rows, int epilogue, void* C, int64_t ldc) {
    DenseGemm g;
    g.A = A;
    g.a_fp32 = b->f32;
    g.lda = lda;
    g.W = static_cast<const uint16_t*>(w.data);
    g.ldw = w.row_stride_bytes / 2;
    g.M = rows;
    g.N = w.rows;
    g.K = w.cols;
    g.epilogue = epilogue;
    g.C = C;
    g.ldc = ldc;
    return g;
}

// prompt rows of a wkv mixer, from its normed inputs in r_hn to r_attn
static int wkv_prompt(BlockStack* b, const ptm_block& L, const LayerRun& run, int M, int64_t pos0, hipStream_t s) {
    const ptm_wkv& m = L.wkv;
    const int hd = m.heads * m.dim, sec = wkv_section(L), es = b->f32 ? 4 : 2;
    const int64_t mix = (int64_t)M * b->wp;  // between the five inputs
    int rc;
    PTM_TRY(token_shift_rows(b->r_hn, run.ring, m.mu, 5, M, pos0, b->wp, b->f32, b->r_mix, s));
    // n rows of `in` from row `first` over input i
    auto section = [&](int i, int first, int n, float* C, int64_t ldc) {
        DenseGemm g = product(b, L.in, static_cast<const uint8_t*>(b->r_mix) + (size_t)(i * mix) * es, b->wp, M, GEMM_F32, C, ldc);
        g.W += (int64_t)first * g.ldw;
        g.N = n;
        return g;
    };
    if (sec == hd && hd % 128 == 0) {
        DenseGemm g = section(0, 0, 4 * hd, b->r_proj, 5 * sec);
        g.section_n = hd;
        g.section_a = mix;
        PTM_TRY(dense_gemm(g, s));
    } else {
        for (int i = 0; i < 4; ++i) PTM_TRY(dense_gemm(section(i, i * hd, hd, b->r_proj + i * sec, 5 * sec), s));
    }
    // few columns: split over K, the sums taken by the tanh
    DenseGemm g = section(4, 4 * hd, m.rank, b->r_h, up64(m.rank));
    g.slab = (int64_t)M * g.ldc;
    g.slab_room = b->r_h_room;
    int slabs = 1;
    PTM_TRY(dense_gemm(g, s, &slabs));
    PTM_TRY(tanh_rows(b->r_h, slabs, g.slab, M, m.rank, b->f32, b->r_low, s));
    DenseGemm decay = product(b, m.w2, b->r_low, up64(m.rank), M, GEMM_DECAY, b->r_proj + 4 * sec, 5 * sec);
    decay.bias = m.w0;
    PTM_TRY(dense_gemm(decay, s));
    WkvRows w{};
    w.proj = b->r_proj;
    w.ld = 5 * sec;
    w.section = sec;
    w.M = M;
    w.heads = m.heads;
    w.dim = m.dim;
    w.u = m.u;
    w.norm = m.norm;
    w.eps = b->cfg.eps;
    w.pos0 = pos0;
    w.state = run.state;
    w.o = b->r_scan;
    w.o_ld = hd;
    w.o_slab = (int64_t)M * hd;
    w.out = b->r_attn;
    w.out_ld = up64(attn_cols(L));
    w.h_last = b->r_hn + (int64_t)(M - 1) * b->wp;
    w.shift = run.ring;
    w.wp = b->wp;
    return wkv_rows(w, b->f32, s);
}

// prompt rows of an attention or latent mixer (and the state-space mixer beside it), from r_xn to r_attn
static int attention_prompt(BlockStack* b, const ptm_block& L, const LayerRun& run, int M, int64_t pos0, hipStream_t s) {
    const bool f32 = b->f32;
    const int es = f32 ? 4 : 2, ldp = up64(qkv_rows(L)), lda = up64(attn_cols(L));
    int rc;
    PTM_TRY(dense_gemm(product(b, L.in, b->r_xn, b->wp, M, GEMM_F32, b->r_proj, ldp), s));
    MixRows m = mix_rows(b, L, run.block, run);
    m.raw = b->r_proj;
    m.ld = ldp;
    m.pos0 = pos0;
    m.q = b->r_q;
    m.q_row = q_cols(L);
    ptm_attention_args a{};
    a.Q = b->r_q;
    a.O = b->r_attn;
    a.q_row = m.q_row;
    a.o_row = lda;
    a.sink = L.sink;
    a.out_scale = L.out_scale;
    if (L.out_gate) {
        a.gate = b->r_proj + gate_row(L);
        a.gate_row = ldp;
        a.gate_head = L.vdim;
    }
    a.rows = M;
    a.heads = L.heads;
    a.dim1 = up8(L.dim);
    a.vdim = up8(L.vdim);
    a.window = L.window;
    a.keep_first = L.keep_first;
    a.pos0 = pos0;
    a.scale = L.scale;
    a.softcap = L.softcap;
    a.fp32 = f32;
    if (latent(L)) {
        if (f32) hipLaunchKernelGGL(latent_prep_rows_kernel<true>, dim3(M), dim3(256), 0, s, m);
        else hipLaunchKernelGGL(latent_prep_rows_kernel<false>, dim3(M), dim3(256), 0, s, m);
        PTM_TRY(launch_status());
        // keys and values of every position some row of the chunk sees
        const int64_t lo = expand_from(L, pos0), row = k_row(L), er = expand_rows(L);
        const uint8_t* cache = static_cast<const uint8_t*>(run.k);
        PTM_TRY(dense_gemm(product(b, L.expand, cache + lo * row * es, row, (int)(pos0 + M - lo), GEMM_ELEM, b->r_kv, er), s));
        a.kv_heads = L.heads;
        a.K1 = b->r_kv;
        a.k1_row = er;
        a.k1_head = a.dim1;
        a.V = static_cast<uint8_t*>(b->r_kv) + (size_t)L.heads * a.dim1 * es;
        a.v_row = er;
        a.v_head = a.vdim;
        a.dim2 = up8(L.rot_dim);
        a.K2 = cache + (lo * row + up8(L.kv_rank)) * es;
        a.k2_row = row;
        a.kv_pos0 = lo;
    } else {
        if (f32) hipLaunchKernelGGL((attention_prep_rows_kernel<true, true>), dim3(M), dim3(256), prep_lds(m), s, m);
        else hipLaunchKernelGGL((attention_prep_rows_kernel<false, false>), dim3(M), dim3(256), prep_lds(m), s, m);
        PTM_TRY(launch_status());
        a.kv_heads = L.kv_heads;
        a.K1 = run.k;
        a.k1_row = m.k_row;
        a.k1_head = a.dim1;
        a.V = run.v;
        a.v_row = m.v_row;
        a.v_head = a.vdim;
    }
    PTM_TRY(attention_rows(a, nullptr, false, s));
    if (has_ssm(L)) {
        SsmRows r{};
        r.m = ssm_shape(L.ssm);
        r.proj = b->r_proj + attn_rows_of(L);
        r.ld = ldp;
        r.M = M;
        r.pos0 = pos0;
        r.eps = b->cfg.eps;
        r.ring = run.ring;
        r.state = run.state;
        r.conv = b->r_conv;
        r.decay = b->r_decay;
        r.y = b->r_scan;
        r.y_slab = (int64_t)M * L.ssm.heads * L.ssm.vdim;
        r.out = static_cast<uint8_t*>(b->r_attn) + (size_t)attn_part(L) * es;
        r.out_ld = lda;
        PTM_TRY(ssm_rows(r, f32, s));
    }
    return PTM_OK;
}

int blocks_rows(BlockStack* b, const int* tokens_host, int M, int64_t pos0, float* trace, hipStream_t s) {
    const ptm_block_config& c = b->cfg;
    const bool f32 = b->f32;
    int rc;
    if (M <= 0 || M > b->rows) return PTM_E_STATE;
    PTM_TRY(hip_status(hipMemcpyAsync(b->r_tokens, tokens_host, 4 * (size_t)M, hipMemcpyHostToDevice, s)));
    const int64_t x_stride = (int64_t)b->rows * b->wp;  // between streams
    if (c.streams > 0)
        hipLaunchKernelGGL(embed_streams_kernel, dim3(M, (b->wp + 511) / 512), dim3(128), 0, s, static_cast<const uint16_t*>(c.embedding.data),
                           c.embedding.row_stride_bytes / 2, b->r_tokens, b->freq, (const int64_t*)nullptr, pos0, c.hidden, b->wp, c.streams, x_stride, b->r_x);
    else
        hipLaunchKernelGGL(embed_bf16_rows_kernel, dim3(M, (b->wp + 511) / 512), dim3(128), 0, s, static_cast<const uint16_t*>(c.embedding.data),
                           c.embedding.row_stride_bytes / 2, b->r_tokens, b->wp, b->r_x, b->r_emb);
    PTM_TRY(launch_status());
    b->r_pend_h = b->r_pend_w = b->r_pend_store = nullptr;
    b->r_branch = 0;
    b->r_slabs = 1;
    const int64_t slab = (int64_t)M * b->wp;
    const float *add0 = nullptr, *add1 = nullptr;
    // the residual rows take in what is pending; their norm (or, gamma NULL, a copy) goes to r_xn unless `only_add`
    // (streams: beta NULL or the layer norm's bias; `fp32_out` leaves the norm in r_hn)
    auto norm = [&](const float* gamma, bool only_add = false, const float* beta = nullptr, bool fp32_out = false) {
        void* xn = only_add ? nullptr : fp32_out ? b->r_hn : b->r_xn;
        if (c.streams > 0) {
            const StreamRows r{b->r_x, c.streams, x_stride, b->r_pend_h, b->r_slabs, slab, b->r_pend_store, branch_blend(b, b->r_branch, false), gamma, beta, xn,
                               c.hidden, b->wp, c.eps};
            if (only_add && !b->r_pend_h) return (int)PTM_OK;
            b->r_pend_h = b->r_pend_store = nullptr;
            b->r_slabs = 1;
            return stream_rows(r, M, f32 || fp32_out, s);
        }
        if (f32) hipLaunchKernelGGL(residual_norm_rows_kernel<true>, dim3(M), dim3(256), 0, s, b->r_x, b->r_pend_h, b->r_slabs, slab, b->r_pend_w, add0, add1, gamma, xn, c.hidden, b->wp, c.eps);
        else hipLaunchKernelGGL(residual_norm_rows_kernel<false>, dim3(M), dim3(256), 0, s, b->r_x, b->r_pend_h, b->r_slabs, slab, b->r_pend_w, add0, add1, gamma, xn, c.hidden, b->wp, c.eps);
        b->r_pend_h = b->r_pend_w = add0 = add1 = nullptr;
        b->r_slabs = 1;
        return launch_status();
    };
    auto branch_out = [&](const ptm_qweight& w, const void* A, const float* post) {
        b->r_pend_h = b->r_h;
        b->r_pend_w = post;
        if (c.streams > 0) b->r_pend_store = branch_store(b, b->r_branch++);
        DenseGemm g = product(b, w, A, up64(w.cols), M, GEMM_F32, b->r_h, b->wp);
        g.slab = slab;
        g.slab_room = b->r_h_room;
        return dense_gemm(g, s, &b->r_slabs);
    };
    for (size_t ri = 0; ri < b->runs.size(); ++ri) {
        const LayerRun& run = b->runs[ri];
        const ptm_block& L = b->blocks[(size_t)run.block];
        if (run.enters_pass >= 0) {
            add0 = run.enters_pass > 0 ? b->r_emb : nullptr;
            add1 = c.loop_step + (int64_t)run.enters_pass * b->wp;
        }
        PTM_TRY(norm(L.norm1, false, L.norm1_bias, wkv(L)));
        if (wkv(L)) PTM_TRY(wkv_prompt(b, L, run, M, pos0, s));
        else PTM_TRY(attention_prompt(b, L, run, M, pos0, s));
        PTM_TRY(branch_out(L.out, b->r_attn, L.norm1b));
        if (L.ff > 0) {
            PTM_TRY(norm(L.norm2, false, L.norm2_bias));
            PTM_TRY(dense_gemm(product(b, L.up, b->r_xn, b->wp, M, L.ff_kind == PTM_FF_SWIGLU ? GEMM_SWIGLU : GEMM_RELU2, b->r_act, up64(L.ff)), s));
            PTM_TRY(branch_out(L.down, b->r_act, L.norm2b));
        }
        if (L.side_gate.data) {
            PTM_TRY(norm(nullptr));
            // few columns: the product is split over K, its sums (in r_h, consumed by the norm above) get the epilogue here
            DenseGemm g = product(b, L.side_gate, b->r_xn, b->wp, M, GEMM_F32, b->r_h, up64(c.side_dim));
            g.slab = (int64_t)M * g.ldc;
            g.slab_room = b->r_h_room;
            int slabs = 1;
            PTM_TRY(dense_gemm(g, s, &slabs));
            const SideRows sr{b->r_h, slabs, g.slab, g.ldc, static_cast<const uint16_t*>(c.side_table.data), c.side_table.row_stride_bytes / 2,
                              L.side_offset, c.side_dim, b->r_tokens, b->r_gate};
            if (f32) hipLaunchKernelGGL(side_rows_kernel<true>, dim3(M), dim3(256), 0, s, sr);
            else hipLaunchKernelGGL(side_rows_kernel<false>, dim3(M), dim3(256), 0, s, sr);
            PTM_TRY(launch_status());
            PTM_TRY(branch_out(L.side_proj, b->r_gate, L.side_norm));
        }
        if (trace) {
            PTM_TRY(norm(nullptr, true));
            PTM_TRY(trace_rows(b, b->r_x, x_stride, M, trace + ri * (size_t)M * (size_t)c.hidden, s));
        }
    }
    if (b->r_slabs > 1 || c.hidden != b->wp || c.streams > 0) PTM_TRY(norm(nullptr, true));  // the head reads finished rows with clear padding
    return PTM_OK;
}
#undef PTM_TRY

}  // namespace ptm

extern "C" int ptm_rope_pairs_host(float* table, int max_seq, const ptm_rotation* rot) {
    if (!table || !rot) return PTM_E_NULL;
    if (max_seq <= 0 || rot->dims <= 0 || (rot->dims & 1) || !(rot->base > 0.0)) return PTM_E_SHAPE;
    const int half = rot->dims / 2;
    std::vector<double> f((size_t)half);
    double amp = 1.0;
    for (int i = 0; i < half; ++i) f[(size_t)i] = std::pow(rot->base, -2.0 * i / rot->dims);
    if (rot->factor > 0.0) {
        const double two_pi = 6.283185307179586476925;
        auto turns = [&](double t) { return rot->dims * std::log(rot->original / (two_pi * t)) / (2.0 * std::log(rot->base)); };
        const double lo = std::fmax(std::floor(turns(rot->fast)), 0.0), hi = std::fmin(std::ceil(turns(rot->slow)), rot->dims - 1.0);
        for (int i = 0; i < half; ++i) {
            const double ramp = std::fmin(std::fmax((i - lo) / std::fmax(hi - lo, 0.001), 0.0), 1.0);
            f[(size_t)i] = f[(size_t)i] / rot->factor * ramp + f[(size_t)i] * (1.0 - ramp);
        }
        amp = 0.1 * std::log(rot->factor) + 1.0;
    }
    for (int p = 0; p < max_seq; ++p)
        for (int i = 0; i < half; ++i) {
            const double a = p * f[(size_t)i];
            table[((size_t)p * half + i) * 2] = (float)(std::cos(a) * amp);
            table[((size_t)p * half + i) * 2 + 1] = (float)(std::sin(a) * amp);
        }
    return PTM_OK;
}
