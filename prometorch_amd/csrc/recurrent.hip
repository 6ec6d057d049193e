// Recurrent mixers: a matrix state per head, kept in fp32 and carried from token to token.
//
//   wkv   o_t = (S + diag(u) k v^T)^T r,  S <- diag(w) S + k v^T          (decay w per key channel and token)
//   ssm   S <- a S + dt B x^T,  y_t = S^T C + D x                         (decay a per head and token; B, C per group of heads)
//
// A state is stored per value column, its key values consecutive and padded: [heads][columns][16 * KPL].  16 lanes share a
// column, KPL key values each, so a wave holds four columns and a read of the state is consecutive.  The columns of a head do not
// depend on each other: the prompt kernels walk the tokens one by one with 16 columns per workgroup, the state in registers, the
// vectors of the next tokens on their way from memory while a tile of tokens is used from LDS.  A sequence's first position starts
// from zeros instead of the stored state, so nothing has to be cleared between sequences.
// What a token needs from earlier ones besides the state (the token shift's vector, the convolution's inputs) lies in rings
// indexed by position; a slot is never read and written by the same launch.
#include "dense.h"

namespace ptm {

__device__ __forceinline__ float softplus_f(float z) { return z > 20.0f ? z : log1pf(expf(z)); }

template <int KPL>
__device__ __forceinline__ void load_keys(float (&s)[KPL], const float* p) {
#pragma unroll
    for (int i = 0; i < KPL; i += 4) {
        const float4 v = *reinterpret_cast<const float4*>(p + i);
        s[i] = v.x; s[i + 1] = v.y; s[i + 2] = v.z; s[i + 3] = v.w;
    }
}
template <int KPL>
__device__ __forceinline__ void store_keys(float* p, const float (&s)[KPL]) {
#pragma unroll
    for (int i = 0; i < KPL; i += 4) *reinterpret_cast<float4*>(p + i) = make_float4(s[i], s[i + 1], s[i + 2], s[i + 3]);
}

// key values per lane for a state of n key channels (0: too many)
static int keys_per_lane(int n) { return n <= 64 ? 4 : n <= 128 ? 8 : n <= 256 ? 16 : n <= 512 ? 32 : 0; }
int64_t recurrent_state_floats(int heads, int keys, int columns) { return (int64_t)heads * columns * 16 * keys_per_lane(keys); }
bool recurrent_supported(int keys) { return keys > 0 && keys_per_lane(keys) > 0; }

// ---- one token ---------------------------------------------------------------------------------
// grid heads, 1024 threads.  64 columns at a time; the low-rank decay product of the head's channels first, the first columns'
// state requested before it.  Output: o over its root mean square, times norm and silu(gate).
template <int KPL>
__global__ __launch_bounds__(1024) void wkv_step_kernel(const WkvStep a) {
    constexpr int KP = 16 * KPL;
    extern __shared__ __align__(16) float s_low[];  // tanh of the low-rank vector, padded to 64
    __shared__ __align__(16) float s_r[KP], s_k[KP], s_u[KP], s_w[KP];
    __shared__ float s_o[KP], s_v[KP], red[16];
    const int tid = threadIdx.x, sub = tid & 15, grp = tid >> 4, h = blockIdx.x, d = a.dim, hd = a.heads * d;
    float* state = a.state + (int64_t)h * d * KP;
    float S[KPL];
    load_keys<KPL>(S, state + (int64_t)min(grp, d - 1) * KP + sub * KPL);
    const int64_t pos = *a.d_past;
    const int rp = (a.rank + 63) & ~63;
    for (int i = tid; i < rp; i += 1024) s_low[i] = i < a.rank ? tanhf(a.proj[4 * (int64_t)hd + i]) : 0.0f;
    for (int i = tid; i < KP; i += 1024) {
        const bool in = i < d;
        const int64_t c = (int64_t)h * d + i;
        s_r[i] = in ? a.proj[c] : 0.0f;
        s_k[i] = in ? a.proj[hd + c] : 0.0f;
        s_v[i] = in ? a.proj[2 * (int64_t)hd + c] : 0.0f;
        s_u[i] = in ? a.u[c] : 0.0f;
        if (!in) s_w[i] = 0.0f;
    }
    __syncthreads();
    for (int c = grp; c < d; c += 64) {
        const uint16_t* row = a.w2 + ((int64_t)h * d + c) * a.w2_ld;
        float t = 0.0f;
        for (int i = sub * 8; i < rp; i += 128) {
            const u32x4 w = *reinterpret_cast<const u32x4*>(row + i);
            const float4 x0 = *reinterpret_cast<const float4*>(s_low + i), x1 = *reinterpret_cast<const float4*>(s_low + i + 4);
            t = fmaf(bf16_lo(w.x), x0.x, t); t = fmaf(bf16_hi(w.x), x0.y, t); t = fmaf(bf16_lo(w.y), x0.z, t); t = fmaf(bf16_hi(w.y), x0.w, t);
            t = fmaf(bf16_lo(w.z), x1.x, t); t = fmaf(bf16_hi(w.z), x1.y, t); t = fmaf(bf16_lo(w.w), x1.z, t); t = fmaf(bf16_hi(w.w), x1.w, t);
        }
        t = sum16(t);
        if (sub == 0) s_w[c] = expf(-expf(t + a.w0[(int64_t)h * d + c]));
    }
    __syncthreads();
    float r[KPL], k[KPL], u[KPL], w[KPL];
    load_keys<KPL>(r, s_r + sub * KPL);
    load_keys<KPL>(k, s_k + sub * KPL);
    load_keys<KPL>(u, s_u + sub * KPL);
    load_keys<KPL>(w, s_w + sub * KPL);
    for (int c0 = 0; c0 < d; c0 += 64) {
        const int c = c0 + grp;
        float* at = state + (int64_t)min(c, d - 1) * KP + sub * KPL;
        if (c0 > 0) load_keys<KPL>(S, at);
        const float v = s_v[min(c, d - 1)];
        float o = 0.0f;
#pragma unroll
        for (int i = 0; i < KPL; ++i) {
            if (pos == 0) S[i] = 0.0f;
            const float kv = k[i] * v;
            o = fmaf(r[i], fmaf(u[i], kv, S[i]), o);
            S[i] = fmaf(w[i], S[i], kv);
        }
        o = sum16(o);
        if (c < d) {
            store_keys<KPL>(at, S);
            if (sub == 0) s_o[c] = o;
        }
    }
    __syncthreads();
    float ss = 0.0f;
    for (int i = tid; i < d; i += 1024) ss = fmaf(s_o[i], s_o[i], ss);
    const float rn = 1.0f / sqrtf(block_sum<16>(ss, red) / (float)d + a.eps);
    for (int i = tid; i < d; i += 1024) {
        const int64_t c = (int64_t)h * d + i;
        a.out[c] = s_o[i] * rn * a.norm[c] * silu_f(a.proj[3 * (int64_t)hd + c]);
    }
}

// the convolution's output for one channel of a token whose own input is x
__device__ __forceinline__ float conv_step(const SsmShape& m, const float* ring, int channels, int ch, int pos, float x) {
    const float* w = m.conv + (int64_t)ch * m.taps;
    float acc = fmaf(w[m.taps - 1], x, m.conv_b[ch]);
    for (int j0 = 1; j0 < m.taps; j0 += 3) {
#pragma unroll
        for (int q = 0; q < 3; ++q) {  // requested together
            const int j = min(j0 + q, m.taps - 1), p = pos - j;
            const float in = ring[(int64_t)(max(p, 0) % m.taps) * channels + ch], t = w[m.taps - 1 - j];
            acc = fmaf(t, j0 + q < m.taps && p >= 0 ? in : 0.0f, acc);
        }
    }
    return silu_f(acc);
}

// grid (heads, ceil(vdim / 16)), 256 threads: convolution, state update, y * silu(z)
template <int KPL>
__global__ __launch_bounds__(256) void ssm_step_kernel(const SsmStep a) {
    constexpr int KP = 16 * KPL;
    __shared__ __align__(16) float s_b[KP], s_c[KP];
    __shared__ float s_x[16];
    const SsmShape& m = a.m;
    const int tid = threadIdx.x, sub = tid & 15, grp = tid >> 4, h = blockIdx.x, N = m.state, g = h / (m.heads / m.groups);
    const int inner = m.heads * m.vdim, channels = inner + 2 * m.groups * N, c = blockIdx.y * 16 + grp;
    float* state = a.state + ((int64_t)h * m.vdim + min(c, m.vdim - 1)) * KP + sub * KPL;
    float S[KPL];
    load_keys<KPL>(S, state);
    const int pos = (int)*a.d_past;
    float* slot = a.ring + (int64_t)(pos % m.taps) * channels;
    const float *z = a.proj, *x = a.proj + inner;  // x, B and C: the convolution's channels
    const bool writer = h % (m.heads / m.groups) == 0 && blockIdx.y == 0;
    for (int i = tid; i < 2 * KP; i += 256) {
        const int n = i % KP;
        float v = 0.0f;
        if (n < N) {
            const int ch = inner + (i < KP ? 0 : m.groups * N) + g * N + n;
            const float in = x[ch];
            v = conv_step(m, a.ring, channels, ch, pos, in);
            if (writer) slot[ch] = in;
        }
        (i < KP ? s_b : s_c)[n] = v;
    }
    if (tid < 16 && (int)blockIdx.y * 16 + tid < m.vdim) {
        const int ch = h * m.vdim + blockIdx.y * 16 + tid;
        const float in = x[ch];
        s_x[tid] = conv_step(m, a.ring, channels, ch, pos, in);
        slot[ch] = in;
    }
    const float dt = softplus_f(a.proj[inner + channels + h] + m.dt_bias[h]), decay = expf(m.neg_a[h] * dt);
    __syncthreads();
    if (c >= m.vdim) return;
    float B[KPL], C[KPL];
    load_keys<KPL>(B, s_b + sub * KPL);
    load_keys<KPL>(C, s_c + sub * KPL);
    const float xv = s_x[grp], dx = dt * xv;
    float y = 0.0f;
#pragma unroll
    for (int i = 0; i < KPL; ++i) {
        if (pos == 0) S[i] = 0.0f;
        S[i] = fmaf(decay, S[i], B[i] * dx);
        y = fmaf(S[i], C[i], y);
    }
    store_keys<KPL>(state, S);
    y = sum16(y);
    const int64_t at = (int64_t)h * m.vdim + c;
    if (sub == 0) a.out[at] = fmaf(m.D[h], xv, y) * silu_f(z[at]);
}

// ---- prompt rows ---------------------------------------------------------------------------------
// tokens per tile: two tiles of three key vectors each in LDS
template <int KPL> constexpr int tile_tokens() { return KPL <= 8 ? 16 : KPL == 16 ? 8 : 4; }

// grid (heads, ceil(dim / 16)), 256 threads
template <int KPL>
__global__ __launch_bounds__(256) void wkv_scan_kernel(const WkvRows a) {
    constexpr int KP = 16 * KPL, TT = tile_tokens<KPL>(), NE = TT * KP / 256;
    __shared__ __align__(16) float s_r[2][TT * KP], s_k[2][TT * KP], s_w[2][TT * KP];
    __shared__ float s_v[2][TT * 16];
    const int tid = threadIdx.x, sub = tid & 15, grp = tid >> 4, h = blockIdx.x, d = a.dim, c = blockIdx.y * 16 + grp;
    if (h == 0 && blockIdx.y == 0)  // the next token's shift reads the last row
        for (int i = tid; i < a.wp; i += 256) a.shift[(a.pos0 + a.M - 1) % 2 * a.wp + i] = a.h_last[i];
    float* state = a.state + ((int64_t)h * d + min(c, d - 1)) * KP + sub * KPL;
    float S[KPL], u[KPL];
    if (a.pos0 > 0) load_keys<KPL>(S, state);
#pragma unroll
    for (int i = 0; i < KPL; ++i) {
        if (a.pos0 == 0) S[i] = 0.0f;
        u[i] = sub * KPL + i < d ? a.u[(int64_t)h * d + sub * KPL + i] : 0.0f;
    }
    // element e of a tile: token e / KP, key channel e % KP; a token past the end leaves the state as it is
    float rr[NE], rk[NE], rw[NE], rv = 0.0f;
    auto fetch = [&](int t0) {
#pragma unroll
        for (int i = 0; i < NE; ++i) {
            const int e = tid + 256 * i, t = t0 + e / KP, k = e % KP;
            const bool in = t < a.M && k < d;
            const int64_t at = (int64_t)min(t, a.M - 1) * a.ld + (int64_t)h * d + min(k, d - 1);
            const float r0 = a.proj[at], k0 = a.proj[at + a.section], w0 = a.w[(int64_t)min(t, a.M - 1) * a.w_ld + (int64_t)h * d + min(k, d - 1)];
            rr[i] = in ? r0 : 0.0f;
            rk[i] = in ? k0 : 0.0f;
            rw[i] = in ? w0 : -INFINITY;
        }
        if (tid < TT * 16) {
            const int t = t0 + tid / 16, cc = blockIdx.y * 16 + tid % 16;
            rv = t < a.M && cc < d ? a.proj[(int64_t)t * a.ld + 2 * a.section + (int64_t)h * d + cc] : 0.0f;
        }
    };
    auto stage = [&](int buf) {
#pragma unroll
        for (int i = 0; i < NE; ++i) {
            const int e = tid + 256 * i;
            s_r[buf][e] = rr[i];
            s_k[buf][e] = rk[i];
            s_w[buf][e] = expf(-expf(rw[i] + a.w0[(int64_t)h * d + min(e % KP, d - 1)]));
        }
        if (tid < TT * 16) s_v[buf][tid] = rv;
    };
    const int tiles = (a.M + TT - 1) / TT;
    fetch(0);
    stage(0);
    __syncthreads();
    for (int tile = 0; tile < tiles; ++tile) {
        const int buf = tile & 1;
        if (tile + 1 < tiles) fetch((tile + 1) * TT);
        float keep = 0.0f;
#pragma unroll 4
        for (int t = 0; t < TT; ++t) {
            float r[KPL], k[KPL], w[KPL], o = 0.0f;
            load_keys<KPL>(r, &s_r[buf][t * KP + sub * KPL]);
            load_keys<KPL>(k, &s_k[buf][t * KP + sub * KPL]);
            load_keys<KPL>(w, &s_w[buf][t * KP + sub * KPL]);
            const float v = s_v[buf][t * 16 + grp];
#pragma unroll
            for (int i = 0; i < KPL; ++i) {
                const float kv = k[i] * v;
                o = fmaf(r[i], fmaf(u[i], kv, S[i]), o);
                S[i] = fmaf(w[i], S[i], kv);
            }
            o = sum16(o);
            keep = sub == t ? o : keep;
        }
        const int t = tile * TT + sub;
        if (sub < TT && t < a.M && c < d) a.o[(int64_t)t * a.o_ld + (int64_t)h * d + c] = keep;
        if (tile + 1 < tiles) stage(buf ^ 1);
        __syncthreads();
    }
    if (c < d) store_keys<KPL>(state, S);
}

// grid rows: each head's o over its root mean square, times norm and silu(gate); a wave per head
template <bool F32>
__global__ __launch_bounds__(256) void wkv_out_rows_kernel(const WkvRows a) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, d = a.dim;
    const float *o = a.o + blockIdx.x * a.o_ld, *g = a.proj + blockIdx.x * a.ld + 3 * a.section;
    for (int h = wave; h < a.heads; h += 4) {
        float ss = 0.0f;
        for (int i = lane; i < d; i += 64) ss = fmaf(o[h * d + i], o[h * d + i], ss);
        const float r = 1.0f / sqrtf(sum64(ss) / (float)d + a.eps);
        for (int i = lane; i < d; i += 64) {
            const int c = h * d + i;
            put_elem<F32>(a.out, blockIdx.x * a.out_ld + c, o[c] * r * a.norm[c] * silu_f(g[c]));
        }
    }
}

// grid (rows, ceil(wp / 1024)): the five inputs h + (h' - h) * mu, [5][rows][wp]
template <bool F32>
__global__ __launch_bounds__(256) void token_shift_rows_kernel(const float* __restrict__ h, const float* __restrict__ shift, const float* __restrict__ mu,
                                                               int n, int64_t pos0, int wp, void* __restrict__ out) {
    const int i = (blockIdx.y * 256 + threadIdx.x) * 4;
    if (i >= wp) return;
    const int64_t row = blockIdx.x;
    const float4 x = *reinterpret_cast<const float4*>(h + row * wp + i);
    float4 p = make_float4(0.f, 0.f, 0.f, 0.f);
    if (row > 0) p = *reinterpret_cast<const float4*>(h + (row - 1) * wp + i);
    else if (pos0 > 0) p = *reinterpret_cast<const float4*>(shift + (pos0 - 1) % 2 * wp + i);
    const float4 d = make_float4(p.x - x.x, p.y - x.y, p.z - x.z, p.w - x.w);
    for (int s = 0; s < n; ++s) {
        const float4 m = *reinterpret_cast<const float4*>(mu + (int64_t)s * wp + i);
        const float4 v = make_float4(fmaf(d.x, m.x, x.x), fmaf(d.y, m.y, x.y), fmaf(d.z, m.z, x.z), fmaf(d.w, m.w, x.w));
        const int64_t at = ((int64_t)s * gridDim.x + row) * wp + i;
        if constexpr (F32) *reinterpret_cast<float4*>(static_cast<float*>(out) + at) = v;
        else *reinterpret_cast<uint2*>(static_cast<uint16_t*>(out) + at) =
                 make_uint2((uint32_t)f_bf16(v.x) | ((uint32_t)f_bf16(v.y) << 16), (uint32_t)f_bf16(v.z) | ((uint32_t)f_bf16(v.w) << 16));
    }
}

// grid rows: tanh of the sum of `slabs` partial products, padded with zeros to ld
template <bool F32>
__global__ __launch_bounds__(64) void tanh_rows_kernel(const float* __restrict__ g, int slabs, int64_t slab, int n, int ld, void* __restrict__ out) {
    for (int i = threadIdx.x; i < ld; i += 64) {
        float v = 0.0f;
        if (i < n)
#pragma unroll 4
            for (int z = 0; z < slabs; ++z) v += g[z * slab + (int64_t)blockIdx.x * ld + i];
        put_elem<F32>(out, (int64_t)blockIdx.x * ld + i, tanhf(v));
    }
}

// grid (rows, ceil(channels / 256)): convolution and silu of x, B and C, [rows][channels]
__global__ __launch_bounds__(256) void ssm_conv_rows_kernel(const SsmRows a) {
    const SsmShape& m = a.m;
    const int inner = m.heads * m.vdim, channels = inner + 2 * m.groups * m.state, ch = blockIdx.y * 256 + threadIdx.x;
    if (ch >= channels) return;
    const int row = blockIdx.x;
    const float *x = a.proj + inner + ch, *w = m.conv + (int64_t)ch * m.taps;
    float acc = m.conv_b[ch];
    for (int j = 0; j < m.taps; ++j) {
        const int64_t p = a.pos0 + row - j;
        if (p < 0) break;
        acc = fmaf(w[m.taps - 1 - j], row >= j ? x[(int64_t)(row - j) * a.ld] : a.ring[p % m.taps * channels + ch], acc);
    }
    a.conv[(int64_t)row * channels + ch] = silu_f(acc);
}

// grid (heads, ceil(vdim / 16)), 256 threads; y takes the place of x in a.conv
template <int KPL>
__global__ __launch_bounds__(256) void ssm_scan_kernel(const SsmRows a) {
    constexpr int KP = 16 * KPL, TT = tile_tokens<KPL>(), NE = TT * KP / 256;
    __shared__ __align__(16) float s_b[2][TT * KP], s_c[2][TT * KP];
    __shared__ float s_x[2][TT * 16], s_a[2][TT], s_dt[2][TT];
    const SsmShape& m = a.m;
    const int tid = threadIdx.x, sub = tid & 15, grp = tid >> 4, h = blockIdx.x, N = m.state, per = m.heads / m.groups, g = h / per;
    const int inner = m.heads * m.vdim, channels = inner + 2 * m.groups * N, c = blockIdx.y * 16 + grp;
    // the ring takes the inputs of the last positions
    for (int j = 0; j < m.taps && j < a.M; ++j) {
        const float* row = a.proj + (int64_t)(a.M - 1 - j) * a.ld + inner;
        float* slot = a.ring + (a.pos0 + a.M - 1 - j) % m.taps * channels;
        if (tid < 16 && (int)blockIdx.y * 16 + tid < m.vdim) slot[h * m.vdim + blockIdx.y * 16 + tid] = row[h * m.vdim + blockIdx.y * 16 + tid];
        if (h % per == 0 && blockIdx.y == 0)
            for (int i = tid; i < 2 * N; i += 256) {
                const int ch = inner + (i < N ? 0 : m.groups * N) + g * N + i % N;
                slot[ch] = row[ch];
            }
    }
    float* state = a.state + ((int64_t)h * m.vdim + min(c, m.vdim - 1)) * KP + sub * KPL;
    float S[KPL];
    if (a.pos0 > 0) load_keys<KPL>(S, state);
    else
#pragma unroll
        for (int i = 0; i < KPL; ++i) S[i] = 0.0f;
    const float *Bp = a.conv + inner + g * N, *Cp = Bp + m.groups * N, dtb = m.dt_bias[h], na = m.neg_a[h], D = m.D[h];
    float rb[NE], rc[NE], rx = 0.0f, rdt = 0.0f;
    auto fetch = [&](int t0) {
#pragma unroll
        for (int i = 0; i < NE; ++i) {
            const int e = tid + 256 * i, t = t0 + e / KP, k = e % KP;
            const bool in = t < a.M && k < N;
            const int64_t at = (int64_t)min(t, a.M - 1) * channels + min(k, N - 1);
            const float b0 = Bp[at], c0 = Cp[at];
            rb[i] = in ? b0 : 0.0f;
            rc[i] = in ? c0 : 0.0f;
        }
        if (tid < TT * 16) {
            const int t = t0 + tid / 16, cc = blockIdx.y * 16 + tid % 16;
            rx = t < a.M && cc < m.vdim ? a.conv[(int64_t)t * channels + h * m.vdim + cc] : 0.0f;
        }
        if (tid < TT) rdt = t0 + tid < a.M ? a.proj[(int64_t)(t0 + tid) * a.ld + inner + channels + h] + dtb : -INFINITY;
    };
    auto stage = [&](int buf) {
#pragma unroll
        for (int i = 0; i < NE; ++i) {
            s_b[buf][tid + 256 * i] = rb[i];
            s_c[buf][tid + 256 * i] = rc[i];
        }
        if (tid < TT * 16) s_x[buf][tid] = rx;
        if (tid < TT) {  // past the end: dt 0, decay 1
            const float dt = softplus_f(rdt);
            s_dt[buf][tid] = dt;
            s_a[buf][tid] = expf(na * dt);
        }
    };
    const int tiles = (a.M + TT - 1) / TT;
    fetch(0);
    stage(0);
    __syncthreads();
    for (int tile = 0; tile < tiles; ++tile) {
        const int buf = tile & 1;
        if (tile + 1 < tiles) fetch((tile + 1) * TT);
        float keep = 0.0f;
#pragma unroll 4
        for (int t = 0; t < TT; ++t) {
            float B[KPL], C[KPL], y = 0.0f;
            load_keys<KPL>(B, &s_b[buf][t * KP + sub * KPL]);
            load_keys<KPL>(C, &s_c[buf][t * KP + sub * KPL]);
            const float x = s_x[buf][t * 16 + grp], decay = s_a[buf][t], dx = s_dt[buf][t] * x;
#pragma unroll
            for (int i = 0; i < KPL; ++i) {
                S[i] = fmaf(decay, S[i], B[i] * dx);
                y = fmaf(S[i], C[i], y);
            }
            y = fmaf(D, x, sum16(y));
            keep = sub == t ? y : keep;
        }
        const int t = tile * TT + sub;
        if (sub < TT && t < a.M && c < m.vdim) a.conv[(int64_t)t * channels + h * m.vdim + c] = keep;
        if (tile + 1 < tiles) stage(buf ^ 1);
        __syncthreads();
    }
    if (c < m.vdim) store_keys<KPL>(state, S);
}

// grid rows: y * silu(z), normed in equal parts, times norm and the branch's scale
template <bool F32>
__global__ __launch_bounds__(256) void ssm_out_rows_kernel(const SsmRows a) {
    __shared__ float red[4];
    const SsmShape& m = a.m;
    const int tid = threadIdx.x, inner = m.heads * m.vdim, channels = inner + 2 * m.groups * m.state, part = inner / m.norm_groups;
    const float *y = a.conv + (int64_t)blockIdx.x * channels, *z = a.proj + blockIdx.x * a.ld;
    constexpr int NS = 16;  // values kept in registers: parts of up to 4096
    for (int p = 0; p < m.norm_groups; ++p) {
        const int c0 = p * part;
        float v[NS], ss = 0.0f;
#pragma unroll
        for (int i = 0; i < NS; ++i) {
            const int c = tid + 256 * i;
            v[i] = c < part ? y[c0 + c] * silu_f(z[c0 + c]) : 0.0f;
            ss = fmaf(v[i], v[i], ss);
        }
        for (int c = tid + 256 * NS; c < part; c += 256) {
            const float t = y[c0 + c] * silu_f(z[c0 + c]);
            ss = fmaf(t, t, ss);
        }
        const float r = 1.0f / sqrtf(block_sum<4>(ss, red) / (float)part + a.eps) * m.scale;
#pragma unroll
        for (int i = 0; i < NS; ++i) {
            const int c = tid + 256 * i;
            if (c < part) put_elem<F32>(a.out, blockIdx.x * a.out_ld + c0 + c, v[i] * r * m.norm[c0 + c]);
        }
        for (int c = tid + 256 * NS; c < part; c += 256)
            put_elem<F32>(a.out, blockIdx.x * a.out_ld + c0 + c, y[c0 + c] * silu_f(z[c0 + c]) * r * m.norm[c0 + c]);
    }
}

// ---- launches ------------------------------------------------------------------------------------
#define PTM_KPL(n, LAUNCH)                                 \
    switch (keys_per_lane(n)) {                            \
        case 4: LAUNCH(4); break;                          \
        case 8: LAUNCH(8); break;                          \
        case 16: LAUNCH(16); break;                        \
        case 32: LAUNCH(32); break;                        \
        default: return PTM_E_UNSUPPORTED;                 \
    }

int wkv_step(const WkvStep& a, hipStream_t s) {
    const size_t lds = (size_t)up64(a.rank) * 4;
    if (a.rank > 8192) return PTM_E_UNSUPPORTED;
#define PTM_RUN(KPL) hipLaunchKernelGGL(wkv_step_kernel<KPL>, dim3(a.heads), dim3(1024), lds, s, a)
    PTM_KPL(a.dim, PTM_RUN)
#undef PTM_RUN
    return launch_status();
}

int ssm_step(const SsmStep& a, hipStream_t s) {
    const dim3 grid(a.m.heads, (a.m.vdim + 15) / 16);
#define PTM_RUN(KPL) hipLaunchKernelGGL(ssm_step_kernel<KPL>, grid, dim3(256), 0, s, a)
    PTM_KPL(a.m.state, PTM_RUN)
#undef PTM_RUN
    return launch_status();
}

int token_shift_rows(const float* h, const float* shift, const float* mu, int n, int rows, int64_t pos0, int wp, bool fp32, void* out, hipStream_t s) {
    const dim3 grid(rows, (wp + 1023) / 1024);
    if (fp32) hipLaunchKernelGGL(token_shift_rows_kernel<true>, grid, dim3(256), 0, s, h, shift, mu, n, pos0, wp, out);
    else hipLaunchKernelGGL(token_shift_rows_kernel<false>, grid, dim3(256), 0, s, h, shift, mu, n, pos0, wp, out);
    return launch_status();
}

int tanh_rows(const float* g, int slabs, int64_t slab, int rows, int n, bool fp32, void* out, hipStream_t s) {
    if (fp32) hipLaunchKernelGGL(tanh_rows_kernel<true>, dim3(rows), dim3(64), 0, s, g, slabs, slab, n, up64(n), out);
    else hipLaunchKernelGGL(tanh_rows_kernel<false>, dim3(rows), dim3(64), 0, s, g, slabs, slab, n, up64(n), out);
    return launch_status();
}

int wkv_rows(const WkvRows& a, bool fp32, hipStream_t s) {
    const dim3 grid(a.heads, (a.dim + 15) / 16);
#define PTM_RUN(KPL) hipLaunchKernelGGL(wkv_scan_kernel<KPL>, grid, dim3(256), 0, s, a)
    PTM_KPL(a.dim, PTM_RUN)
#undef PTM_RUN
    if (fp32) hipLaunchKernelGGL(wkv_out_rows_kernel<true>, dim3(a.M), dim3(256), 0, s, a);
    else hipLaunchKernelGGL(wkv_out_rows_kernel<false>, dim3(a.M), dim3(256), 0, s, a);
    return launch_status();
}

int ssm_rows(const SsmRows& a, bool fp32, hipStream_t s) {
    const SsmShape& m = a.m;
    const int channels = m.heads * m.vdim + 2 * m.groups * m.state;
    hipLaunchKernelGGL(ssm_conv_rows_kernel, dim3(a.M, (channels + 255) / 256), dim3(256), 0, s, a);
    const dim3 grid(m.heads, (m.vdim + 15) / 16);
#define PTM_RUN(KPL) hipLaunchKernelGGL(ssm_scan_kernel<KPL>, grid, dim3(256), 0, s, a)
    PTM_KPL(m.state, PTM_RUN)
#undef PTM_RUN
    if (fp32) hipLaunchKernelGGL(ssm_out_rows_kernel<true>, dim3(a.M), dim3(256), 0, s, a);
    else hipLaunchKernelGGL(ssm_out_rows_kernel<false>, dim3(a.M), dim3(256), 0, s, a);
    return launch_status();
}
#undef PTM_KPL

}  // namespace ptm
