// Recurrent mixers: a matrix state per head, kept in fp32 and carried from token to token.
//
//   wkv   o_t = (S + diag(u) k v^T)^T r,  S <- diag(w) S + k v^T          (decay w per key channel and token)
//   ssm   S <- a S + dt B x^T,  y_t = S^T C + D x                         (decay a per head and token; B, C per group of heads)
//
// A state is stored per value column, its key values consecutive and padded: [heads][columns][16 * KPL].
// One token: 16 lanes share a column, KPL key values each, so a wave holds four columns and a read of the state is consecutive.
// Prompt rows: neither the columns nor the keys of a state depend on each other, only the sum over the keys does.  A lane is a value
// column and a wave has KPL keys of 64 columns in registers, so what belongs to a key (r, k, w; B, C) is one value for the whole
// wave: it is loaded once into a row of 16 lanes and broadcast as a DPP operand of the arithmetic, three instructions per key and
// token.  A workgroup's four waves add their sums through LDS; up to four workgroups share a head and leave partial sums, which the
// row kernel behind the scan adds.  The next tile's vectors are on their way while a tile of tokens is used.
// A sequence's first position starts from zeros instead of the stored state, so nothing has to be cleared between sequences.
// What a token needs from earlier ones besides the state (the token shift's vector, the convolution's inputs) lies in rings
// indexed by position; a slot is never read and written by the same launch.
#include "dense.h"

#include <type_traits>

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

// f(integral constants 0 .. N - 1)
template <int N, int I = 0, typename F>
__device__ __forceinline__ void static_for(F f) {
    if constexpr (I < N) {
        f(std::integral_constant<int, I>{});
        static_for<N, I + 1>(f);
    }
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
// workgroups that share the keys of a head, four waves of KPL keys each
static int key_groups(int keys) { return (keys + 4 * keys_per_lane(keys) - 1) / (4 * keys_per_lane(keys)); }

// value of lane N of each row of 16 lanes, as an operand of the next instruction
template <int N>
__device__ __forceinline__ float row_lane(float v) { return dpp_f<0x150 + N>(v); }

// The waves' sums of a tile of TT tokens (s_o [4][TT][64]), on their way from LDS while the next tile is used: this wave's rows
// wave, wave + 4, ...
template <int TT>
struct TileSums {
    float v[TT / 4][4];
    __device__ __forceinline__ void read(const float (*s_o)[TT][64]) {
        const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
#pragma unroll
        for (int q = 0; q < TT / 4; ++q)
#pragma unroll
            for (int w = 0; w < 4; ++w) v[q][w] = s_o[w][wave + 4 * q][lane];
    }
    __device__ __forceinline__ void store(float* out, int64_t ld, int t0, int M, int columns) const {
        const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
#pragma unroll
        for (int q = 0; q < TT / 4; ++q) {
            const int t = t0 + wave + 4 * q;
            if (t < M && lane < columns) out[(int64_t)t * ld + lane] = (v[q][0] + v[q][1]) + (v[q][2] + v[q][3]);
        }
    }
};

// Four keys of 64 columns take four tokens: o += S^T r, S <- diag(w) S + k v^T.  p[t]: a row of lanes [r | k | w | -], four each.
// (One block, because the compiler does not fold the broadcasts into the multiply-adds; the wait states are for p.)
#define PTM_DPP(n) " row_newbcast:" n " row_mask:0xf bank_mask:0xf\n\t"
#define PTM_WKV_TOKEN(O, P, V)                                   \
    "v_fmac_f32_dpp %" O ", %" P ", %0" PTM_DPP("0")             \
    "v_mul_f32_dpp %0, %" P ", %0" PTM_DPP("8")                  \
    "v_fmac_f32_dpp %" O ", %" P ", %1" PTM_DPP("1")             \
    "v_mul_f32_dpp %1, %" P ", %1" PTM_DPP("9")                  \
    "v_fmac_f32_dpp %" O ", %" P ", %2" PTM_DPP("2")             \
    "v_mul_f32_dpp %2, %" P ", %2" PTM_DPP("10")                 \
    "v_fmac_f32_dpp %" O ", %" P ", %3" PTM_DPP("3")             \
    "v_mul_f32_dpp %3, %" P ", %3" PTM_DPP("11")                 \
    "v_fmac_f32_dpp %0, %" P ", %" V PTM_DPP("4")                \
    "v_fmac_f32_dpp %1, %" P ", %" V PTM_DPP("5")                \
    "v_fmac_f32_dpp %2, %" P ", %" V PTM_DPP("6")                \
    "v_fmac_f32_dpp %3, %" P ", %" V PTM_DPP("7")
__device__ __forceinline__ void wkv_keys4(float* s, float (&o)[4], float p0, float p1, float p2, float p3, float v0, float v1, float v2, float v3) {
    asm("s_nop 1\n\t" PTM_WKV_TOKEN("4", "8", "12") PTM_WKV_TOKEN("5", "9", "13") PTM_WKV_TOKEN("6", "10", "14") PTM_WKV_TOKEN("7", "11", "15")
        : "+&v"(s[0]), "+&v"(s[1]), "+&v"(s[2]), "+&v"(s[3]), "+&v"(o[0]), "+&v"(o[1]), "+&v"(o[2]), "+&v"(o[3])
        : "v"(p0), "v"(p1), "v"(p2), "v"(p3), "v"(v0), "v"(v1), "v"(v2), "v"(v3));
}

// grid (heads, key groups * ceil(dim / 64)), 256 threads.  Without the bonus, which the row kernel behind it adds.
template <int KPL>
__global__ __launch_bounds__(256, 1) void wkv_scan_kernel(const WkvRows a) {
    constexpr int KP = 16 * KPL, Q = KPL / 4, TT = Q < 4 ? 16 / Q : 4;  // Q rows of [r | k | w] of four keys per token
    __shared__ float s_o[2][4][TT][64];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), h = blockIdx.x, d = a.dim;
    const int kg = blockIdx.y % a.groups, c0 = blockIdx.y / a.groups * 64, c = min(c0 + lane, d - 1), k0 = (4 * kg + wave) * KPL;
    if (h == 0 && blockIdx.y == 0)  // the next token's shift reads the last row
        for (int i = tid; i < a.wp; i += 256) a.shift[(a.pos0 + a.M - 1) % 2 * a.wp + i] = a.h_last[i];
    float* state = a.state + ((int64_t)h * d + c) * KP + k0;
    float S[KPL];
    if (a.pos0 > 0) load_keys<KPL>(S, state);
    else
#pragma unroll
        for (int i = 0; i < KPL; ++i) S[i] = 0.0f;
    // lane j of a row of lanes: r (0..3), k (4..7), w (8..11) of key k0 + 4 q + j % 4; keys past the end, and lanes 12..15, are zeros
    const uint32_t step = (uint32_t)a.ld * 4, bytes = (uint32_t)a.M * step, part = (lane >> 2) & 3;
    const __amdgpu_buffer_rsrc_t rs = make_rsrc(a.proj, (int)bytes);
    uint32_t off[Q];
#pragma unroll
    for (int q = 0; q < Q; ++q) {
        const int key = k0 + 4 * q + (lane & 3);
        off[q] = key < d && part < 3 ? (uint32_t)((part == 2 ? 4 : part) * a.section + h * d + key) * 4 : bytes;
    }
    const uint32_t voff = (uint32_t)(2 * a.section + h * d + c) * 4;
    struct Tile { float p[TT][Q], v[TT]; } A, B;
    const uint32_t last = bytes - step;
    auto fetch = [&](Tile& x, int t0) {  // rows past the last repeat it and are not used
        uint32_t row = min((uint32_t)t0 * step, last);
#pragma unroll
        for (int t = 0; t < TT; ++t) {
#pragma unroll
            for (int q = 0; q < Q; ++q) x.p[t][q] = __uint_as_float(__builtin_amdgcn_raw_buffer_load_b32(rs, off[q], row, 0));
            x.v[t] = __uint_as_float(__builtin_amdgcn_raw_buffer_load_b32(rs, voff, row, 0));
            row = min(row + step, last);
        }
        issue_order_fence();
    };
    float* out = a.o + kg * a.o_slab + (int64_t)h * d + c0;
    TileSums<TT> sums;
    auto run = [&](Tile& x, int t0, int buf) {  // a token past the last leaves the state as it is
        if (t0 > 0) sums.read(s_o[buf ^ 1]);
        if (t0 + TT > a.M) {
            const float keep = part == 2 ? 1.0f : 0.0f;
#pragma unroll
            for (int t = 0; t < TT; ++t)
                if (t0 + t >= a.M)
#pragma unroll
                    for (int q = 0; q < Q; ++q) x.p[t][q] = keep;
        }
#pragma unroll
        for (int t = 0; t < TT; t += 4) {
            float o[4] = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int q = 0; q < Q; ++q)
                wkv_keys4(S + 4 * q, o, x.p[t][q], x.p[t + 1][q], x.p[t + 2][q], x.p[t + 3][q], x.v[t], x.v[t + 1], x.v[t + 2], x.v[t + 3]);
#pragma unroll
            for (int i = 0; i < 4; ++i) s_o[buf][wave][t + i][lane] = o[i];
        }
        if (t0 > 0) sums.store(out, a.o_ld, t0 - TT, a.M, d - c0);
        __syncthreads();
    };
    fetch(A, 0);
    int t0 = 0;
    for (;; t0 += 2 * TT) {
        fetch(B, t0 + TT);
        run(A, t0, 0);
        if (t0 + TT >= a.M) break;
        fetch(A, t0 + 2 * TT);
        run(B, t0 + TT, 1);
        if (t0 + 2 * TT >= a.M) { t0 += TT; break; }
    }
    sums.read(s_o[t0 / TT & 1]);
    sums.store(out, a.o_ld, t0, a.M, d - c0);
    if (c0 + lane < d) store_keys<KPL>(state, S);
}

// grid (rows, ceil(heads / 4)), a wave per head: o = the scan's sums + the bonus; over its root mean square, times norm and
// silu(gate).  NV: values per lane.
template <bool F32, int NV>
__global__ __launch_bounds__(256) void wkv_out_rows_kernel(const WkvRows a) {
    const int lane = threadIdx.x & 63, h = blockIdx.y * 4 + (threadIdx.x >> 6), d = a.dim;
    if (h >= a.heads) return;
    const float *p = a.proj + blockIdx.x * a.ld + h * d, *o = a.o + blockIdx.x * a.o_ld + h * d;
    float x[NV][4], v[NV], g[NV], n[NV], b[NV];
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int e = min(lane + 64 * i, d - 1);
#pragma unroll
        for (int z = 0; z < 4; ++z) x[i][z] = z < a.groups ? o[z * a.o_slab + e] : 0.0f;
        v[i] = p[2 * a.section + e];
        g[i] = p[3 * a.section + e];
        n[i] = a.norm[h * d + e];
        b[i] = p[e] * a.u[h * d + e] * p[a.section + e];
    }
    float bonus = 0.0f, ss = 0.0f;
#pragma unroll
    for (int i = 0; i < NV; ++i) bonus += lane + 64 * i < d ? b[i] : 0.0f;
    bonus = sum64(bonus);
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        v[i] = lane + 64 * i < d ? fmaf(bonus, v[i], (x[i][0] + x[i][1]) + (x[i][2] + x[i][3])) : 0.0f;
        ss = fmaf(v[i], v[i], ss);
    }
    const float r = 1.0f / sqrtf(sum64(ss) / (float)d + a.eps);
#pragma unroll
    for (int i = 0; i < NV; ++i)
        if (lane + 64 * i < d) put_elem<F32>(a.out, blockIdx.x * a.out_ld + h * d + lane + 64 * i, v[i] * r * n[i] * silu_f(g[i]));
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

// grid (ceil(rows / 8), ceil(channels / 256) + 1): convolution and silu of x, B and C, [rows][channels], eight rows per thread;
// the last column of workgroups leaves decay and dt, [rows][2][heads]
constexpr int CONV_ROWS = 8;
__global__ __launch_bounds__(256) void ssm_conv_rows_kernel(const SsmRows a) {
    const SsmShape& m = a.m;
    const int inner = m.heads * m.vdim, channels = inner + 2 * m.groups * m.state, r0 = blockIdx.x * CONV_ROWS, rows = min(CONV_ROWS, a.M - r0);
    if (blockIdx.y == gridDim.y - 1) {
        for (int i = threadIdx.x; i < rows * m.heads; i += 256) {
            const int64_t row = r0 + i / m.heads;
            const int h = i % m.heads;
            const float dt = softplus_f(a.proj[row * a.ld + inner + channels + h] + m.dt_bias[h]);
            a.decay[row * 2 * m.heads + h] = expf(m.neg_a[h] * dt);
            a.decay[(row * 2 + 1) * m.heads + h] = dt;
        }
        return;
    }
    const int ch = blockIdx.y * 256 + threadIdx.x;
    if (ch >= channels) return;
    const float *x = a.proj + inner + ch, *w = m.conv + (int64_t)ch * m.taps, bias = m.conv_b[ch];
    auto input = [&](int row) {  // of row r0 + row, also of rows and positions before
        const int64_t p = a.pos0 + r0 + row;
        return r0 + row >= 0 ? x[(int64_t)min(r0 + row, a.M - 1) * a.ld] : p >= 0 ? a.ring[p % m.taps * channels + ch] : 0.0f;
    };
    float* out = a.conv + (int64_t)r0 * channels + ch;
    if (m.taps <= 4) {
        float in[CONV_ROWS + 3], t[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) t[j] = j < m.taps ? w[m.taps - 1 - j] : 0.0f;
#pragma unroll
        for (int i = 0; i < CONV_ROWS + 3; ++i) in[i] = 3 - i < m.taps ? input(i - 3) : 0.0f;
#pragma unroll
        for (int r = 0; r < CONV_ROWS; ++r)
            if (r < rows) out[(int64_t)r * channels] = silu_f(fmaf(t[3], in[r], fmaf(t[2], in[r + 1], fmaf(t[1], in[r + 2], fmaf(t[0], in[r + 3], bias)))));
    } else {
        for (int r = 0; r < rows; ++r) {
            float acc = bias;
            for (int j = 0; j < m.taps; ++j) acc = fmaf(w[m.taps - 1 - j], input(r - j), acc);
            out[(int64_t)r * channels] = silu_f(acc);
        }
    }
}

// Four keys of 64 columns take four tokens: S <- decay S + B dx, y += C S.  p[t]: a row of lanes with B at lanes B0 .. and C at
// C0 .. .
#define PTM_DECAY(S, D) "v_mul_f32 %" S ", %" D ", %" S "\n\t"
#define PTM_SSM_TAKE(P, X)                                       \
    "v_fmac_f32_dpp %0, %" P ", %" X PTM_DPP("%20")              \
    "v_fmac_f32_dpp %1, %" P ", %" X PTM_DPP("%21")              \
    "v_fmac_f32_dpp %2, %" P ", %" X PTM_DPP("%22")              \
    "v_fmac_f32_dpp %3, %" P ", %" X PTM_DPP("%23")
#define PTM_SSM_GIVE(Y, P, S, C) "v_fmac_f32_dpp %" Y ", %" P ", %" S PTM_DPP("%" C)
#define PTM_SSM_GIVE_NEXT(Y, P, D)                               \
    PTM_SSM_GIVE(Y, P, "0", "24") PTM_DECAY("0", D)              \
    PTM_SSM_GIVE(Y, P, "1", "25") PTM_DECAY("1", D)              \
    PTM_SSM_GIVE(Y, P, "2", "26") PTM_DECAY("2", D)              \
    PTM_SSM_GIVE(Y, P, "3", "27") PTM_DECAY("3", D)
template <int B0, int C0>
__device__ __forceinline__ void ssm_keys4(float* s, float (&y)[4], float p0, float p1, float p2, float p3, const float* decay, const float* dx) {
    asm(PTM_DECAY("0", "12") PTM_DECAY("1", "12") PTM_DECAY("2", "12") PTM_DECAY("3", "12")
        PTM_SSM_TAKE("8", "16") PTM_SSM_GIVE_NEXT("4", "8", "13")
        PTM_SSM_TAKE("9", "17") PTM_SSM_GIVE_NEXT("5", "9", "14")
        PTM_SSM_TAKE("10", "18") PTM_SSM_GIVE_NEXT("6", "10", "15")
        PTM_SSM_TAKE("11", "19")
        PTM_SSM_GIVE("7", "11", "0", "24") PTM_SSM_GIVE("7", "11", "1", "25") PTM_SSM_GIVE("7", "11", "2", "26") PTM_SSM_GIVE("7", "11", "3", "27")
        : "+&v"(s[0]), "+&v"(s[1]), "+&v"(s[2]), "+&v"(s[3]), "+&v"(y[0]), "+&v"(y[1]), "+&v"(y[2]), "+&v"(y[3])
        : "v"(p0), "v"(p1), "v"(p2), "v"(p3), "v"(decay[0]), "v"(decay[1]), "v"(decay[2]), "v"(decay[3]), "v"(dx[0]), "v"(dx[1]), "v"(dx[2]), "v"(dx[3]),
          "n"(B0), "n"(B0 + 1), "n"(B0 + 2), "n"(B0 + 3), "n"(C0), "n"(C0 + 1), "n"(C0 + 2), "n"(C0 + 3));
}

// grid (heads, key groups * ceil(vdim / 64)), 256 threads; without the skip D x, which the row kernel behind it adds
template <int KPL>
__global__ __launch_bounds__(256, 1) void ssm_scan_kernel(const SsmRows a) {
    constexpr int KP = 16 * KPL, KQ = KPL < 8 ? KPL : 8, Q = KPL / KQ, TT = 16 / Q;  // Q rows of [B | C] of KQ keys per token
    constexpr int NG = (TT + 7) / 8;
    __shared__ float s_o[2][4][TT][64];
    const SsmShape& m = a.m;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), h = blockIdx.x, N = m.state;
    const int per = m.heads / m.groups, g = h / per, inner = m.heads * m.vdim, channels = inner + 2 * m.groups * N;
    const int kg = blockIdx.y % a.key_groups, c0 = blockIdx.y / a.key_groups * 64, c = min(c0 + lane, m.vdim - 1), k0 = (4 * kg + wave) * KPL;
    // the ring takes the inputs of the last positions
    for (int j = 0; j < m.taps && j < a.M; ++j) {
        const float* row = a.proj + (int64_t)(a.M - 1 - j) * a.ld + inner;
        float* slot = a.ring + (a.pos0 + a.M - 1 - j) % m.taps * channels;
        if (kg == 0 && wave == 0 && c0 + lane < m.vdim) slot[h * m.vdim + c] = row[h * m.vdim + c];
        if (h % per == 0 && blockIdx.y == 0)
            for (int i = tid; i < 2 * N; i += 256) {
                const int ch = inner + (i < N ? 0 : m.groups * N) + g * N + i % N;
                slot[ch] = row[ch];
            }
    }
    float* state = a.state + ((int64_t)h * m.vdim + c) * KP + k0;
    float S[KPL];
    if (a.pos0 > 0) load_keys<KPL>(S, state);
    else
#pragma unroll
        for (int i = 0; i < KPL; ++i) S[i] = 0.0f;
    // lane j of a row of lanes: B (j < KQ) or C (KQ <= j < 2 KQ) of key k0 + KQ q + j % KQ; the other lanes, and keys past the end,
    // are zeros
    const uint32_t step = (uint32_t)channels * 4, bytes = (uint32_t)a.M * step;
    const __amdgpu_buffer_rsrc_t rs = make_rsrc(a.conv, (int)bytes);
    uint32_t off[Q];
#pragma unroll
    for (int q = 0; q < Q; ++q) {
        const int j = lane & 15, key = k0 + KQ * q + j % KQ;
        off[q] = key < N && j < 2 * KQ ? (uint32_t)(inner + (j < KQ ? 0 : m.groups * N) + g * N + key) * 4 : bytes;
    }
    const uint32_t xoff = (uint32_t)(h * m.vdim + c) * 4;
    const float* dsrc = a.decay + (lane & 8 ? m.heads : 0) + h;
    struct Tile { float p[TT][Q], x[TT], d[NG]; } A, B;
    const uint32_t last = bytes - step;
    auto fetch = [&](Tile& x, int t0) {  // rows past the last repeat it and are not used
        uint32_t row = min((uint32_t)t0 * step, last);
#pragma unroll
        for (int i = 0; i < NG; ++i) x.d[i] = dsrc[(int64_t)min(t0 + 8 * i + (lane & 7), a.M - 1) * 2 * m.heads];  // decay, then dt, of eight tokens
#pragma unroll
        for (int t = 0; t < TT; ++t) {
#pragma unroll
            for (int q = 0; q < Q; ++q) x.p[t][q] = __uint_as_float(__builtin_amdgcn_raw_buffer_load_b32(rs, off[q], row, 0));
            x.x[t] = __uint_as_float(__builtin_amdgcn_raw_buffer_load_b32(rs, xoff, row, 0));
            row = min(row + step, last);
        }
        issue_order_fence();
    };
    float* out = a.y + kg * a.y_slab + h * m.vdim + c0;
    TileSums<TT> sums;
    auto run = [&](Tile& x, int t0, int buf) {  // a token past the last leaves the state as it is
        if (t0 > 0) sums.read(s_o[buf ^ 1]);
        float decay[TT], dx[TT];
        static_for<TT>([&](auto T) {
            constexpr int t = decltype(T)::value;
            decay[t] = row_lane<t % 8>(x.d[t / 8]);
            dx[t] = row_lane<8 + t % 8>(x.d[t / 8]) * x.x[t];
        });
        if (t0 + TT > a.M) {
#pragma unroll
            for (int t = 0; t < TT; ++t)
                if (t0 + t >= a.M) {
                    decay[t] = 1.0f;
                    dx[t] = 0.0f;
                }
        }
#pragma unroll
        for (int t = 0; t < TT; t += 4) {
            float y[4] = {0.0f, 0.0f, 0.0f, 0.0f};
            static_for<KPL / 4>([&](auto I) {
                constexpr int i = 4 * decltype(I)::value, b0 = i % KQ, q = i / KQ;
                ssm_keys4<b0, KQ + b0>(S + i, y, x.p[t][q], x.p[t + 1][q], x.p[t + 2][q], x.p[t + 3][q], decay + t, dx + t);
            });
#pragma unroll
            for (int i = 0; i < 4; ++i) s_o[buf][wave][t + i][lane] = y[i];
        }
        if (t0 > 0) sums.store(out, inner, t0 - TT, a.M, m.vdim - c0);
        __syncthreads();
    };
    fetch(A, 0);
    int t0 = 0;
    for (;; t0 += 2 * TT) {
        fetch(B, t0 + TT);
        run(A, t0, 0);
        if (t0 + TT >= a.M) break;
        fetch(A, t0 + 2 * TT);
        run(B, t0 + TT, 1);
        if (t0 + 2 * TT >= a.M) { t0 += TT; break; }
    }
    sums.read(s_o[t0 / TT & 1]);
    sums.store(out, inner, t0, a.M, m.vdim - c0);
    if (c0 + lane < m.vdim) store_keys<KPL>(state, S);
}

// grid rows: (the scan's sums + D x) * silu(z), normed in equal parts, times norm and the branch's scale
template <bool F32>
__global__ __launch_bounds__(256) void ssm_out_rows_kernel(const SsmRows a) {
    __shared__ float red[4];
    const SsmShape& m = a.m;
    const int tid = threadIdx.x, inner = m.heads * m.vdim, channels = inner + 2 * m.groups * m.state, part = inner / m.norm_groups;
    const float *y = a.y + (int64_t)blockIdx.x * inner, *x = a.conv + (int64_t)blockIdx.x * channels, *z = a.proj + blockIdx.x * a.ld;
    auto value = [&](int c) {
        float s[4];
#pragma unroll
        for (int k = 0; k < 4; ++k) s[k] = k < a.key_groups ? y[k * a.y_slab + c] : 0.0f;
        return fmaf(m.D[c / m.vdim], x[c], (s[0] + s[1]) + (s[2] + s[3])) * silu_f(z[c]);
    };
    constexpr int NS = 16;  // values kept in registers: parts of up to 4096
    for (int p = 0; p < m.norm_groups; ++p) {
        const int c0 = p * part;
        float v[NS], ss = 0.0f;
#pragma unroll
        for (int i = 0; i < NS; ++i) {
            const int c = tid + 256 * i;
            v[i] = c < part ? value(c0 + c) : 0.0f;
            ss = fmaf(v[i], v[i], ss);
        }
        for (int c = tid + 256 * NS; c < part; c += 256) {
            const float t = value(c0 + c);
            ss = fmaf(t, t, ss);
        }
        const float r = 1.0f / sqrtf(block_sum<4>(ss, red) / (float)part + a.eps) * m.scale;
#pragma unroll
        for (int i = 0; i < NS; ++i) {
            const int c = tid + 256 * i;
            if (c < part) put_elem<F32>(a.out, blockIdx.x * a.out_ld + c0 + c, v[i] * r * m.norm[c0 + c]);
        }
        for (int c = tid + 256 * NS; c < part; c += 256) put_elem<F32>(a.out, blockIdx.x * a.out_ld + c0 + c, value(c0 + c) * r * m.norm[c0 + c]);
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

int64_t scan_slabs(int keys) { return key_groups(keys); }

int wkv_rows(WkvRows a, bool fp32, hipStream_t s) {
    if (!recurrent_supported(a.dim)) return PTM_E_UNSUPPORTED;
    a.groups = key_groups(a.dim);
    const dim3 grid(a.heads, a.groups * ((a.dim + 63) / 64));
#define PTM_RUN(KPL) hipLaunchKernelGGL(wkv_scan_kernel<KPL>, grid, dim3(256), 0, s, a)
    PTM_KPL(a.dim, PTM_RUN)
#undef PTM_RUN
    const dim3 out_grid(a.M, (a.heads + 3) / 4);
#define PTM_RUN(NV)                                                                                                  \
    if (fp32) hipLaunchKernelGGL((wkv_out_rows_kernel<true, NV>), out_grid, dim3(256), 0, s, a);                     \
    else hipLaunchKernelGGL((wkv_out_rows_kernel<false, NV>), out_grid, dim3(256), 0, s, a)
    if (a.dim <= 64) { PTM_RUN(1); }
    else if (a.dim <= 128) { PTM_RUN(2); }
    else { PTM_RUN(8); }
#undef PTM_RUN
    return launch_status();
}

int ssm_rows(SsmRows a, bool fp32, hipStream_t s) {
    const SsmShape& m = a.m;
    if (!recurrent_supported(m.state)) return PTM_E_UNSUPPORTED;
    const int channels = m.heads * m.vdim + 2 * m.groups * m.state;
    a.key_groups = key_groups(m.state);
    hipLaunchKernelGGL(ssm_conv_rows_kernel, dim3((a.M + CONV_ROWS - 1) / CONV_ROWS, (channels + 255) / 256 + 1), dim3(256), 0, s, a);
    const dim3 grid(m.heads, a.key_groups * ((m.vdim + 63) / 64));
#define PTM_RUN(KPL) hipLaunchKernelGGL(ssm_scan_kernel<KPL>, grid, dim3(256), 0, s, a)
    PTM_KPL(m.state, PTM_RUN)
#undef PTM_RUN
    if (fp32) hipLaunchKernelGGL(ssm_out_rows_kernel<true>, dim3(a.M), dim3(256), 0, s, a);
    else hipLaunchKernelGGL(ssm_out_rows_kernel<false>, dim3(a.M), dim3(256), 0, s, a);
    return launch_status();
}
#undef PTM_KPL

}  // namespace ptm
