// Softmax attention of the block decoders: head sizes, value sizes, softcap, sliding window with kept first positions and
// keys in two parts (one shared by all heads) are parameters.
//
//   attention_rows_kernel    one wave per (row, head), fp32 arithmetic, fp32 or bfloat16 rows: fp32 decoders, and head sizes
//                            the matrix-core kernels have no class for
//   attention_mfma_kernel    prompt rows, bfloat16: a workgroup owns one kv head and 128 query vectors, walks the visible
//                            keys in tiles of 64 through LDS; S^T = K . Q^T, online softmax in the accumulator layout,
//                            O^T += V^T . P^T with P as two bfloat16 terms (16 bits of the fp32 weights)
//   decode_mfma_kernel       one token, bfloat16 caches: workgroup = (16 query heads of a kv head, share of the visible
//                            64-position chunks), a wave per 16 positions; q and p as two bfloat16 terms each; partial results
//                            per share, merged by the next launch.  A latent mixer's step is this kernel with one kv head whose
//                            values are the first part of its keys.
#include "dense.h"

namespace ptm {

typedef __bf16 at_b8 __attribute__((ext_vector_type(8)));
typedef short at_s4 __attribute__((ext_vector_type(4)));
typedef float at_f4 __attribute__((ext_vector_type(4)));
typedef float at_f16 __attribute__((ext_vector_type(16)));
constexpr float LOG2E = 1.44269504088896340736f;

// ds_read_b64_tr_b16: within each group of 16 lanes, lane i passes the address of four 16-bit values (row i / 4 of a 4-row
// block, columns 4 (i % 4) .. +3 of a 16-column block) and receives column i of the four rows.
__device__ __forceinline__ at_s4 lds_tr16(const uint8_t* p) {
    typedef __attribute__((address_space(3))) at_s4 lds_s4;
    return __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4*)p);
}
__device__ __forceinline__ short bf_bits(float f) { return (short)f_bf16(f); }
__device__ __forceinline__ float bf_val(short s) { return bf16_f((uint16_t)s); }
// cap * tanh(s / cap); 1 - 2 / (e^2y + 1) ends at +-1 for large arguments
__device__ __forceinline__ float soft_cap(float s, float cap, float inv_cap) {
    const float e = __builtin_amdgcn_exp2f(s * inv_cap * (2.0f * LOG2E));
    return cap * (1.0f - 2.0f * __builtin_amdgcn_rcpf(e + 1.0f));
}

// factor of value dimension v of a finished result: output gate and scale
__device__ __forceinline__ float out_factor(const ptm_attention_args& a, int64_t row, int head, int v) {
    const float s = a.out_scale != 0.0f ? a.out_scale : 1.0f;
    return a.gate && v < a.gate_head ? s * sigmoid_f(a.gate[row * a.gate_row + (int64_t)head * a.gate_head + v]) : s;
}

__device__ __forceinline__ bool sees(int64_t pos, int64_t key, int window, int keep) {
    return key <= pos && (window <= 0 || pos - key < window || key < keep);
}

// ---- plain kernel ------------------------------------------------------------------------------
template <bool F32>
__device__ __forceinline__ float dot8(const void* p, int64_t at, const float* q) {
    float s = 0.0f;
    if constexpr (F32) {
        const float4 a = *reinterpret_cast<const float4*>(static_cast<const float*>(p) + at);
        const float4 b = *reinterpret_cast<const float4*>(static_cast<const float*>(p) + at + 4);
        s = fmaf(a.x, q[0], s); s = fmaf(a.y, q[1], s); s = fmaf(a.z, q[2], s); s = fmaf(a.w, q[3], s);
        s = fmaf(b.x, q[4], s); s = fmaf(b.y, q[5], s); s = fmaf(b.z, q[6], s); s = fmaf(b.w, q[7], s);
    } else {
        const uint4 u = *reinterpret_cast<const uint4*>(static_cast<const uint16_t*>(p) + at);
        s = fmaf(bf16_lo(u.x), q[0], s); s = fmaf(bf16_hi(u.x), q[1], s); s = fmaf(bf16_lo(u.y), q[2], s); s = fmaf(bf16_hi(u.y), q[3], s);
        s = fmaf(bf16_lo(u.z), q[4], s); s = fmaf(bf16_hi(u.z), q[5], s); s = fmaf(bf16_lo(u.w), q[6], s); s = fmaf(bf16_hi(u.w), q[7], s);
    }
    return s;
}

// grid (rows, heads), one wave; lanes take keys for the scores and value dimensions for the sum
template <bool F32, bool Q32, int VT>
__global__ __launch_bounds__(64) void attention_rows_kernel(const ptm_attention_args a, const int64_t* d_past) {
    extern __shared__ __align__(16) float s_q[];  // [dim1 + dim2], then 64 weights
    const int lane = threadIdx.x, row = blockIdx.x, h = blockIdx.y, g = h / (a.heads / a.kv_heads), dq = a.dim1 + a.dim2;
    float* s_p = s_q + dq;
    const int64_t pos = (d_past ? *d_past : a.pos0) + row;
    const int64_t qo = (int64_t)row * a.q_row + (int64_t)h * dq;
    for (int i = lane; i < dq; i += 64) s_q[i] = get_elem<Q32>(a.Q, qo + i);
    __syncthreads();
    float acc[VT];
#pragma unroll
    for (int t = 0; t < VT; ++t) acc[t] = 0.0f;
    float m = a.sink ? a.sink[h] : -INFINITY, l = a.sink ? 1.0f : 0.0f;
    const int64_t lo = a.window > 0 && pos - a.window + 1 > 0 ? pos - a.window + 1 : 0;
    const int64_t keep = a.keep_first < lo ? a.keep_first : lo;
    for (int part = 0; part < 2; ++part) {
        const int64_t k_begin = part ? lo : 0, k_end = part ? pos + 1 : keep;
        for (int64_t k0 = k_begin; k0 < k_end; k0 += 64) {
            const int n = (int)(k_end - k0 < 64 ? k_end - k0 : 64);
            const int64_t at = k0 - a.kv_pos0;
            float s = -INFINITY;
            if (lane < n) {
                float t = 0.0f;
                const int64_t k1 = (at + lane) * a.k1_row + (int64_t)g * a.k1_head, k2 = (at + lane) * a.k2_row;
                for (int i = 0; i < a.dim1; i += 8) t += dot8<F32>(a.K1, k1 + i, s_q + i);
                for (int i = 0; i < a.dim2; i += 8) t += dot8<F32>(a.K2, k2 + i, s_q + a.dim1 + i);
                s = t * a.scale;
                if (a.softcap > 0.0f) s = a.softcap * tanhf(s / a.softcap);
            }
            const float mn = fmaxf(m, max64(s)), corr = expf(m - mn), p = expf(s - mn);
            m = mn;
            l = l * corr + sum64(p);
            __syncthreads();
            s_p[lane] = p;
            __syncthreads();
#pragma unroll
            for (int t = 0; t < VT; ++t) acc[t] *= corr;
            for (int k = 0; k < n; ++k) {
                const float pk = s_p[k];
                const int64_t v = (at + k) * a.v_row + (int64_t)g * a.v_head;
#pragma unroll
                for (int t = 0; t < VT; ++t)
                    if (lane + 64 * t < a.vdim) acc[t] = fmaf(pk, get_elem<F32>(a.V, v + lane + 64 * t), acc[t]);
            }
        }
    }
    const float inv = 1.0f / l;
    const int64_t o = (int64_t)row * a.o_row + (int64_t)h * a.vdim;
#pragma unroll
    for (int t = 0; t < VT; ++t)
        if (lane + 64 * t < a.vdim) put_elem<Q32>(a.O, o + lane + 64 * t, acc[t] * inv * out_factor(a, row, h, lane + 64 * t));
}

template <bool F32, bool Q32>
static int rows_launch(const ptm_attention_args& a, const int64_t* d_past, hipStream_t s) {
    const dim3 grid(a.rows, a.heads), block(64);
    const size_t lds = (size_t)(a.dim1 + a.dim2 + 64) * 4;
    const int vt = (a.vdim + 63) / 64;
    if (vt <= 1) hipLaunchKernelGGL((attention_rows_kernel<F32, Q32, 1>), grid, block, lds, s, a, d_past);
    else if (vt <= 2) hipLaunchKernelGGL((attention_rows_kernel<F32, Q32, 2>), grid, block, lds, s, a, d_past);
    else if (vt <= 8) hipLaunchKernelGGL((attention_rows_kernel<F32, Q32, 8>), grid, block, lds, s, a, d_past);
    else hipLaunchKernelGGL((attention_rows_kernel<F32, Q32, 32>), grid, block, lds, s, a, d_past);
    return launch_status();
}

// ---- prompt rows on the matrix cores --------------------------------------------------------------
// v_mfma_f32_32x32x16_bf16: A: lane l holds row l % 32, summation indices 8 (l / 32) + 0..7; B: column l % 32, the same
// indices; C: column l % 32, rows 8 (r / 4) + 4 (l / 32) + r % 4.  The 16 keys of a P.V step are the ones the lane already
// holds in its S^T accumulator, in that order.
template <int DQ, int DV>
__global__ __launch_bounds__(256, DQ <= 192 && DV <= 128 ? 2 : 1) void attention_mfma_kernel(const ptm_attention_args a) {
    constexpr int KS = DQ / 16, DT = DV / 32, KP = DQ * 2 + 16, VP = DV * 2 + 64;
    __shared__ __align__(16) uint8_t s_k[64 * KP];
    __shared__ __align__(16) uint8_t s_v[64 * VP];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), j = lane & 31, kh = lane >> 5;
    const int per = a.heads / a.kv_heads, dq = a.dim1 + a.dim2;
    int sh = 0;  // a row takes 1 << sh slots (heads) of a wave's 32 query vectors
    while ((1 << sh) < per && sh < 5) ++sh;
    const int htiles = (per + 31) / 32, rpw = 32 >> sh, bm = 4 * rpw;
    // longest row blocks first, all kv heads of a block together
    const int gh = blockIdx.x % (a.kv_heads * htiles), g = gh / htiles, ht = gh % htiles;
    const int m_base = ((a.rows + bm - 1) / bm - 1 - (int)blockIdx.x / (a.kv_heads * htiles)) * bm;
    const int slot = (j & ((1 << sh) - 1)) + 32 * ht, row = m_base + wave * rpw + (j >> sh);
    const bool live = slot < per && row < a.rows;
    const int row_c = row < a.rows ? row : a.rows - 1, head = g * per + (slot < per ? slot : per - 1);
    const int64_t pos = a.pos0 + row_c;

    at_b8 qf[KS];
    {
        const uint16_t* src = static_cast<const uint16_t*>(a.Q) + (int64_t)row_c * a.q_row + (int64_t)head * dq + 8 * kh;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
            u32x4 v = {0, 0, 0, 0};
            if (16 * ks + 8 * kh < dq) v = *reinterpret_cast<const u32x4*>(src + 16 * ks);
            qf[ks] = __builtin_bit_cast(at_b8, v);
        }
    }
    at_f16 acc[DT];
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
#pragma unroll
        for (int r = 0; r < 16; ++r) acc[dt][r] = 0.0f;
    // the two lane halves of a query add their sums at the end: one of them holds the sink
    float m_run = a.sink ? a.sink[head] * LOG2E : -INFINITY, l_run = a.sink && kh == 0 ? 1.0f : 0.0f;

    const int64_t p_min = a.pos0 + m_base, p_max = a.pos0 + (m_base + bm < a.rows ? m_base + bm : a.rows) - 1;
    const int wt0 = a.window > 0 && p_min - a.window + 1 > 0 ? (int)((p_min - a.window + 1) / 64) : 0;
    const int kt = (a.keep_first + 63) / 64, nk = a.window > 0 ? (kt < wt0 ? kt : wt0) : 0;
    const int ntiles = nk + (int)(p_max / 64) - wt0 + 1;
    auto tile_at = [&](int i) { return i < nk ? i : wt0 + i - nk; };

    // A thread stages 16-byte pieces of rows tid / 8 and tid / 8 + 32, columns 8 (tid % 8) + 64 g; pieces past the key or value
    // size are zeros.
    constexpr int GK = DQ / 64, GV = DV / 64;
    const int r0 = tid >> 3, c0 = (tid & 7) * 8;
    const uint16_t* kp[GK];
    const uint16_t* vp[GV];
    uint32_t kstr[GK];
#pragma unroll
    for (int i = 0; i < GK; ++i) {
        const int c = c0 + 64 * i;
        kp[i] = c < a.dim1 ? static_cast<const uint16_t*>(a.K1) + (int64_t)g * a.k1_head + c
                           : c < dq ? static_cast<const uint16_t*>(a.K2) + (c - a.dim1) : nullptr;
        kstr[i] = (uint32_t)(c < a.dim1 ? a.k1_row : a.k2_row);
    }
#pragma unroll
    for (int i = 0; i < GV; ++i) {
        const int c = c0 + 64 * i;
        vp[i] = c < a.vdim ? static_cast<const uint16_t*>(a.V) + (int64_t)g * a.v_head + c : nullptr;
    }
    u32x4 kreg[2 * GK], vreg[2 * GV];
    const int key_last = (int)(p_max - a.kv_pos0);
    // keys past the last visible one repeat it, keys before the array its first; both are masked
    auto key_of = [&](int tile, int r) {
        const int key = (int)((int64_t)tile * 64 - a.kv_pos0) + r;
        return (uint32_t)max(min(key, key_last), 0);
    };
    auto fetch_k = [&](int tile) {
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const uint32_t key = key_of(tile, r0 + 32 * u);
#pragma unroll
            for (int i = 0; i < GK; ++i) {
                kreg[GK * u + i] = u32x4{0, 0, 0, 0};
                if (kp[i]) kreg[GK * u + i] = *reinterpret_cast<const u32x4*>(kp[i] + (uint64_t)key * kstr[i]);
            }
        }
    };
    auto fetch_v = [&](int tile) {
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const uint32_t key = key_of(tile, r0 + 32 * u);
#pragma unroll
            for (int i = 0; i < GV; ++i) {
                vreg[GV * u + i] = u32x4{0, 0, 0, 0};
                if (vp[i]) vreg[GV * u + i] = *reinterpret_cast<const u32x4*>(vp[i] + (uint64_t)key * (uint32_t)a.v_row);
            }
        }
    };
    const float sc2 = a.scale * LOG2E, inv_cap = a.softcap > 0.0f ? 1.0f / a.softcap : 0.0f;
    fetch_k(tile_at(0));
    fetch_v(tile_at(0));
    for (int it = 0; it < ntiles; ++it) {
        const int64_t k0 = (int64_t)tile_at(it) * 64;
        __syncthreads();  // every wave has finished reading the previous tile
#pragma unroll
        for (int u = 0; u < 2; ++u) {
#pragma unroll
            for (int i = 0; i < GK; ++i) *reinterpret_cast<u32x4*>(s_k + (r0 + 32 * u) * KP + (c0 + 64 * i) * 2) = kreg[GK * u + i];
#pragma unroll
            for (int i = 0; i < GV; ++i) *reinterpret_cast<u32x4*>(s_v + (r0 + 32 * u) * VP + (c0 + 64 * i) * 2) = vreg[GV * u + i];
        }
        __syncthreads();
        const int next = tile_at(it + 1 < ntiles ? it + 1 : it);
        fetch_k(next);
        issue_order_fence();
        at_f16 sc[2];
#pragma unroll
        for (int u = 0; u < 2; ++u) {
#pragma unroll
            for (int r = 0; r < 16; ++r) sc[u][r] = 0.0f;
#pragma unroll
            for (int ks = 0; ks < KS; ++ks) {
                const at_b8 ka = *reinterpret_cast<const at_b8*>(s_k + (32 * u + j) * KP + (16 * ks + 8 * kh) * 2);
                sc[u] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(ka, qf[ks], sc[u], 0, 0, 0);
            }
        }
        issue_order_fence();
        fetch_v(next);
        issue_order_fence();
        if (a.softcap > 0.0f) {
#pragma unroll
            for (int u = 0; u < 2; ++u)
#pragma unroll
                for (int r = 0; r < 16; ++r) sc[u][r] = soft_cap(sc[u][r] * a.scale, a.softcap, inv_cap) * LOG2E;
        } else {
#pragma unroll
            for (int u = 0; u < 2; ++u)
#pragma unroll
                for (int r = 0; r < 16; ++r) sc[u][r] *= sc2;
        }
        // a tile some query of the workgroup does not see whole (workgroup-uniform)
        const bool whole = k0 + 63 <= p_min && (a.window <= 0 || p_max - k0 < a.window || k0 + 63 < a.keep_first);
        if (!whole) {
            issue_order_fence();  // keeps this a branch
            const int last = (int)(pos - k0 < 64 ? pos - k0 : 64);                                        // keys up to here
            const int64_t f64 = a.window > 0 ? pos - a.window + 1 - k0 : 0;
            const int first = (int)(f64 < 0 ? 0 : f64 < 64 ? f64 : 64);                                   // window from here
            const int kept = (int)(a.keep_first - k0 < 0 ? 0 : a.keep_first - k0 < 64 ? a.keep_first - k0 : 64);  // kept below here
#pragma unroll
            for (int u = 0; u < 2; ++u)
#pragma unroll
                for (int r = 0; r < 16; ++r) {
                    const int o = 32 * u + 8 * (r >> 2) + 4 * kh + (r & 3);
                    sc[u][r] = o <= last && (o >= first || o < kept) ? sc[u][r] : -INFINITY;
                }
        }
        float mx = sc[0][0];
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int r = 0; r < 16; ++r) mx = fmaxf(mx, sc[u][r]);
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        const float m_new = fmaxf(m_run, mx), ms = m_new == -INFINITY ? 0.0f : m_new;  // nothing visible yet
        const float corr = __builtin_amdgcn_exp2f(m_run - ms);
        float psum = 0.0f;
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int r = 0; r < 16; ++r) {
                sc[u][r] = __builtin_amdgcn_exp2f(sc[u][r] - ms);
                psum += sc[u][r];
            }
        l_run = fmaf(l_run, corr, psum);
        if (__builtin_amdgcn_ballot_w64(m_new != m_run) != 0) {
#pragma unroll
            for (int dt = 0; dt < DT; ++dt)
#pragma unroll
                for (int r = 0; r < 16; ++r) acc[dt][r] *= corr;
        }
        m_run = m_new;
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int ks = 0; ks < 2; ++ks) {
                at_b8 hi, lo;
#pragma unroll
                for (int i = 0; i < 8; ++i) {
                    const float p = sc[u][8 * ks + i];
                    hi[i] = (__bf16)p;
                    lo[i] = (__bf16)(p - (float)hi[i]);
                }
#pragma unroll
                for (int dt = 0; dt < DT; ++dt) {
                    const uint8_t* vrow = s_v + (32 * u + 16 * ks + 4 * kh + ((lane & 15) >> 2)) * VP + (32 * dt + (j & 16) + 4 * (lane & 3)) * 2;
                    const at_s4 v0 = lds_tr16(vrow), v1 = lds_tr16(vrow + 8 * VP);
                    typedef short s8 __attribute__((ext_vector_type(8)));
                    const at_b8 va = __builtin_bit_cast(at_b8, (s8){v0[0], v0[1], v0[2], v0[3], v1[0], v1[1], v1[2], v1[3]});
                    acc[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(va, hi, acc[dt], 0, 0, 0);
                    acc[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(va, lo, acc[dt], 0, 0, 0);
                }
            }
    }
    const float inv = 1.0f / (l_run + __shfl_xor(l_run, 32, 64));
    if (!live) return;
    uint16_t* dst = static_cast<uint16_t*>(a.O) + (int64_t)row * a.o_row + (int64_t)head * a.vdim + 4 * kh;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
#pragma unroll
        for (int q = 0; q < 4; ++q)
            if (32 * dt + 8 * q < a.vdim) {
                float v0 = acc[dt][4 * q] * inv, v1 = acc[dt][4 * q + 1] * inv, v2 = acc[dt][4 * q + 2] * inv, v3 = acc[dt][4 * q + 3] * inv;
                if (a.gate || a.out_scale != 0.0f) {
                    const int v = 32 * dt + 8 * q + 4 * kh;
                    v0 *= out_factor(a, row, head, v);
                    v1 *= out_factor(a, row, head, v + 1);
                    v2 *= out_factor(a, row, head, v + 2);
                    v3 *= out_factor(a, row, head, v + 3);
                }
                *reinterpret_cast<uint2*>(dst + 32 * dt + 8 * q) =
                    make_uint2((uint32_t)f_bf16(v0) | ((uint32_t)f_bf16(v1) << 16), (uint32_t)f_bf16(v2) | ((uint32_t)f_bf16(v3) << 16));
            }
}

template <int DQ, int DV>
static int mfma_launch(const ptm_attention_args& a, hipStream_t s) {
    const int per = a.heads / a.kv_heads;
    int sh = 0;
    while ((1 << sh) < per && sh < 5) ++sh;
    const int bm = 4 * (32 >> sh), htiles = (per + 31) / 32;
    const dim3 grid((unsigned)((a.rows + bm - 1) / bm * a.kv_heads * htiles));
    hipLaunchKernelGGL((attention_mfma_kernel<DQ, DV>), grid, dim3(256), 0, s, a);
    return launch_status();
}

static int check_args(const ptm_attention_args& a) {
    if (!a.Q || !a.K1 || !a.V || !a.O || (a.dim2 > 0 && !a.K2)) return PTM_E_NULL;
    if (a.rows <= 0 || a.heads <= 0 || a.kv_heads <= 0 || a.heads % a.kv_heads || a.dim1 <= 0 || a.dim2 < 0 || a.vdim <= 0 ||
        a.window < 0 || a.keep_first < 0 || a.pos0 < 0 || a.kv_pos0 < 0)
        return PTM_E_SHAPE;
    if (a.gate && a.gate_head <= 0) return PTM_E_SHAPE;
    if (a.kv_pos0 > 0 && (a.keep_first > 0 || a.window <= 0 || a.pos0 - a.window + 1 < a.kv_pos0)) return PTM_E_RANGE;  // a visible key before the array
    if ((a.dim1 | a.dim2 | a.vdim | a.k1_row | a.k1_head | a.k2_row | a.v_row | a.v_head | a.q_row | a.o_row) & 7) return PTM_E_ALIGN;
    if (!aligned16(a.Q) || !aligned16(a.K1) || !aligned16(a.V) || !aligned16(a.O) || (a.K2 && !aligned16(a.K2))) return PTM_E_ALIGN;
    if (a.dim1 + a.dim2 > 8192 || a.vdim > 2048) return PTM_E_UNSUPPORTED;
    return PTM_OK;
}

int attention_rows(const ptm_attention_args& a, const int64_t* d_past, bool q_fp32_out_fp32, hipStream_t s) {
    const int rc = check_args(a);
    if (rc != PTM_OK) return rc;
    const int dq = a.dim1 + a.dim2;
    if (a.fp32) return rows_launch<true, true>(a, d_past, s);
    if (q_fp32_out_fp32) return rows_launch<false, true>(a, d_past, s);
    if (a.pos0 + a.rows > 0x7fffffff || ((a.k1_row | a.k2_row | a.v_row) >> 31)) return PTM_E_UNSUPPORTED;
    if (d_past || dq > 256 || a.vdim > 256) return rows_launch<false, false>(a, d_past, s);
    if (dq <= 64 && a.vdim <= 64) return mfma_launch<64, 64>(a, s);
    if (dq <= 128 && a.vdim <= 64) return mfma_launch<128, 64>(a, s);
    if (dq <= 128 && a.vdim <= 128) return mfma_launch<128, 128>(a, s);
    if (dq <= 192 && a.vdim <= 128) return mfma_launch<192, 128>(a, s);
    return mfma_launch<256, 256>(a, s);
}

// ---- one decode token on the matrix cores ---------------------------------------------------------
// v_mfma_f32_16x16x32_bf16: A: lane l holds row l % 16, summation indices 8 (l / 16) + 0..7; B: column l % 16 alike; C: column
// l % 16, rows 4 (l / 16) + r.  A wave scores 16 of a chunk's 64 positions (S^T = K . Q^T); the weights, in the layout the
// scores were left in, go to all waves through LDS and each sums a quarter of the value dimensions over the whole chunk
// (O^T = V^T . P^T): two tiles of 16 positions make the 32 summation indices, each lane's eight being the positions
// 4 (l / 16) + 0..3 of either tile.
// RAW: q, k, v arrive un-normed; every workgroup norms and rotates its heads' q (behind the requests for its first keys and
// values), the one that holds the newest position also the key, takes it (and the value) from LDS and appends both rows to the
// caches.  Otherwise q is ready as two bfloat16 planes [2][heads][dim1 + dim2].
__device__ __forceinline__ float sumsq_part(const float* p, int n) {  // this thread's share of 256
    float s = 0.0f;
    if (((n | (int)(reinterpret_cast<uintptr_t>(p) >> 2)) & 3) == 0) {
#pragma unroll 4
        for (int i = threadIdx.x; i < n / 4; i += 256) {
            const float4 v = reinterpret_cast<const float4*>(p)[i];
            s = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, s))));
        }
    } else {
#pragma unroll 4
        for (int i = threadIdx.x; i < n; i += 256) s = fmaf(p[i], p[i], s);
    }
    return s;
}

template <int DQ, int DV, bool RAW, bool V_IS_K>
__global__ __launch_bounds__(256, 1) void decode_mfma_kernel(const DecodeAttention d, int splits) {
    constexpr int KS = DQ / 32, DW = DV / 64, QP = DQ * 2 + 16, VP = DV * 2 + 32, PV = V_IS_K ? 1 : DV / 32;
    __shared__ __align__(16) uint8_t s_q[2][16 * QP];
    __shared__ __align__(16) uint8_t s_v[64 * VP];
    __shared__ __align__(16) at_s4 s_p[2][4][64];
    __shared__ __align__(16) uint16_t s_newk[RAW ? DQ : 8], s_newv[RAW ? DV : 8];
    __shared__ float s_m[4][16], s_l[4][16], red[4], s_rq[RAW ? 17 : 1];
    const ptm_attention_args& a = d.a;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), j = lane & 15, rg = lane >> 4;
    const int per = a.heads / a.kv_heads, tiles = (per + 15) / 16, dq = a.dim1 + a.dim2;
    const int split = blockIdx.x, g = blockIdx.y / tiles, h0 = g * per + 16 * (blockIdx.y % tiles);
    const int nh = min(16, (g + 1) * per - h0);
    constexpr int QN = RAW ? 1 : 2 * 16 * DQ / 8 / 256;  // 16-byte pieces of the q planes per thread
    u32x4 qr[QN];
    if constexpr (!RAW) {  // requested first: they do not depend on the position
#pragma unroll
        for (int i = 0; i < QN; ++i) {
            const int p = tid + 256 * i, t = p / (2 * DQ), h = p / (DQ / 8) % 16, c = p % (DQ / 8) * 8;
            qr[i] = u32x4{0, 0, 0, 0};
            if (h < nh && c < dq)
                qr[i] = *reinterpret_cast<const u32x4*>(static_cast<const uint16_t*>(a.Q) + ((int64_t)t * a.heads + h0 + h) * dq + c);
        }
    }
    const int64_t past = *d.d_past;
    const int64_t lo = a.window > 0 && past - a.window + 1 > 0 ? past - a.window + 1 : 0;
    const int wc0 = (int)(lo / 64), kc = (a.keep_first + 63) / 64, nk = a.window > 0 ? (kc < wc0 ? kc : wc0) : 0;
    const int total = nk + (int)(past / 64) - wc0 + 1;
    if (split >= total) {  // nothing to do: the merge gives this share weight 0
        if (tid < nh) {
            d.pM[(int64_t)split * a.heads + h0 + tid] = -INFINITY;
            d.pL[(int64_t)split * a.heads + h0 + tid] = 0.0f;
        }
        return;
    }
    const bool newest = (total - 1) % splits == split;  // this workgroup's share holds the newest position
    u32x4 ka[KS], vv[PV];
    const int ntrips = (total - split + splits - 1) / splits;
    auto first_key = [&](int c) { return (int64_t)(c < nk ? c : wc0 + c - nk) * 64 + 16 * wave; };
    auto fetch = [&](int64_t k0) {  // positions past the newest repeat it and are masked
        const int64_t kpos = k0 + j < past ? k0 + j : past;
        const uint16_t* k1 = static_cast<const uint16_t*>(a.K1) + kpos * a.k1_row + (int64_t)g * a.k1_head;
        const uint16_t* k2 = static_cast<const uint16_t*>(a.K2) + kpos * a.k2_row - a.dim1;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
            const int col = 32 * ks + 8 * rg;
            ka[ks] = u32x4{0, 0, 0, 0};
            if (col < dq) ka[ks] = *reinterpret_cast<const u32x4*>((col < a.dim1 ? k1 : k2) + col);
        }
        if constexpr (!V_IS_K) {
#pragma unroll
            for (int i = 0; i < PV; ++i) {
                const int q = lane + 64 * i, r = q / (DV / 8), col = (q % (DV / 8)) * 8;
                const int64_t vpos = k0 + r < past ? k0 + r : past;
                vv[i] = u32x4{0, 0, 0, 0};
                if (col < a.vdim) vv[i] = *reinterpret_cast<const u32x4*>(static_cast<const uint16_t*>(a.V) + vpos * a.v_row + (int64_t)g * a.v_head + col);
            }
        }
    };
    fetch(first_key(split));
    if constexpr (RAW) {
        const int nq = a.heads * d.dim, nkv = a.kv_heads * d.dim;
        const float *rawk = d.raw + nq, *cs = d.rope + past * d.rot_dims;
        auto turned = [&](const float* p, const float* w, float r, int c) {
            const float v = p[c] * r * w[c];
            if (c >= d.rot_dims) return v;
            const float o = p[c ^ 1] * r * w[c ^ 1], co = cs[2 * (c >> 1)], sn = cs[2 * (c >> 1) + 1];
            return (c & 1) ? v * co + o * sn : v * co - o * sn;
        };
        float pk = 0.0f, rq = 0.0f;
        if (d.head_norm) {  // a wave per head; [16]: the key head
            for (int h = wave; h < nh + (newest ? 1 : 0); h += 4) {
                const float* p = h < nh ? d.raw + (h0 + h) * d.dim : rawk + g * d.dim;
                float ss = 0.0f;
#pragma unroll 4
                for (int c = lane; c < d.dim; c += 64) ss = fmaf(p[c], p[c], ss);
                ss = sum64(ss);
                if (lane == 0) s_rq[h < nh ? h : 16] = 1.0f / sqrtf(ss / (float)d.dim + d.eps);
            }
            __syncthreads();
        } else {
            const float pq = sumsq_part(d.raw, nq);
            pk = newest ? sumsq_part(rawk, nkv) : 0.0f;
            rq = 1.0f / sqrtf(block_sum<4>(pq, red) / (float)nq + d.eps);
        }
#pragma unroll 2
        for (int i = tid; i < nh * DQ; i += 256) {
            const int h = i / DQ, c = i % DQ;
            const float v = c < d.dim ? turned(d.raw + (h0 + h) * d.dim, d.q_norm + (h0 + h) * d.dim, d.head_norm ? s_rq[h] : rq, c) : 0.0f;
            const short hi = bf_bits(v);
            *reinterpret_cast<short*>(s_q[0] + h * QP + c * 2) = hi;
            *reinterpret_cast<short*>(s_q[1] + h * QP + c * 2) = bf_bits(v - bf_val(hi));
        }
        for (int i = tid; i < (16 - nh) * (DQ / 2); i += 256) {  // columns without a head
            const int h = nh + i / (DQ / 2), c = i % (DQ / 2);
            *reinterpret_cast<uint32_t*>(s_q[0] + h * QP + c * 4) = 0;
            *reinterpret_cast<uint32_t*>(s_q[1] + h * QP + c * 4) = 0;
        }
        if (newest) {
            const float rk = d.head_norm ? s_rq[16] : 1.0f / sqrtf(block_sum<4>(pk, red) / (float)nkv + d.eps);
            const float* rawv = rawk + (d.values_are_keys ? 0 : nkv) + g * d.vdim_true;
            const bool writer = blockIdx.y % tiles == 0;
            for (int c = tid; c < DQ; c += 256) {
                const uint16_t b = f_bf16(c < d.dim ? turned(rawk + g * d.dim, d.k_norm + g * d.dim, rk, c) : 0.0f);
                s_newk[c] = b;
                if (writer && c < a.dim1) static_cast<uint16_t*>(d.k_cache)[past * a.k1_row + (int64_t)g * a.k1_head + c] = b;
            }
            for (int c = tid; c < DV; c += 256) {
                const uint16_t b = f_bf16(c < d.vdim_true ? rawv[c] : 0.0f);
                s_newv[c] = b;
                if (writer && c < a.vdim) static_cast<uint16_t*>(d.v_cache)[past * a.v_row + (int64_t)g * a.v_head + c] = b;
            }
        }
    } else {
#pragma unroll
        for (int i = 0; i < QN; ++i) {
            const int p = tid + 256 * i, t = p / (2 * DQ), h = p / (DQ / 8) % 16, c = p % (DQ / 8) * 8;
            *reinterpret_cast<u32x4*>(s_q[t] + h * QP + c * 2) = qr[i];
        }
    }
    __syncthreads();
    // the fragment of q's plane t for columns 32 ks + 8 rg .. of head j
    auto q_frag = [&](int t, int ks) { return *reinterpret_cast<const at_b8*>(s_q[t] + j * QP + (32 * ks + 8 * rg) * 2); };
    at_f4 acc[DW];
#pragma unroll
    for (int i = 0; i < DW; ++i) acc[i] = at_f4{0.f, 0.f, 0.f, 0.f};
    float m_run = -INFINITY, l_run = 0.0f;
    const float sc2 = a.scale * LOG2E, inv_cap = a.softcap > 0.0f ? 1.0f / a.softcap : 0.0f;
    uint8_t* sv = s_v + 16 * wave * VP;
    for (int trip = 0; trip < ntrips; ++trip) {
        const int64_t k0 = first_key(split + trip * splits);
        if (trip > 0) {
            fetch(k0);
            __syncthreads();  // every wave has finished with the previous chunk's values and weights
        }
        if constexpr (V_IS_K) {
#pragma unroll
            for (int ks = 0; ks < DV / 32; ++ks) *reinterpret_cast<u32x4*>(sv + j * VP + (32 * ks + 8 * rg) * 2) = ka[ks];
        } else {
#pragma unroll
            for (int i = 0; i < PV; ++i) {
                const int q = lane + 64 * i, r = q / (DV / 8), col = (q % (DV / 8)) * 8;
                if constexpr (RAW) {
                    if (k0 + r >= past) vv[i] = *reinterpret_cast<const u32x4*>(s_newv + col);
                }
                *reinterpret_cast<u32x4*>(sv + r * VP + col * 2) = vv[i];
            }
        }
        if constexpr (RAW) {
            if (k0 + j >= past) {
#pragma unroll
                for (int ks = 0; ks < KS; ++ks) ka[ks] = *reinterpret_cast<const u32x4*>(s_newk + 32 * ks + 8 * rg);
            }
        }
        at_f4 s1 = {0.f, 0.f, 0.f, 0.f}, s2 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
            const at_b8 k8 = __builtin_bit_cast(at_b8, ka[ks]);
            s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k8, q_frag(0, ks), s1, 0, 0, 0);
            s2 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k8, q_frag(1, ks), s2, 0, 0, 0);
        }
        float sc[4], mx = -INFINITY;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            float v = s1[r] + s2[r];
            v = a.softcap > 0.0f ? soft_cap(v * a.scale, a.softcap, inv_cap) * LOG2E : v * sc2;
            sc[r] = sees(past, k0 + 4 * rg + r, a.window, a.keep_first) ? v : -INFINITY;
            mx = fmaxf(mx, sc[r]);
        }
        mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        if (rg == 0) s_m[wave][j] = mx;
        __syncthreads();
        const float m_new = fmaxf(m_run, fmaxf(fmaxf(s_m[0][j], s_m[1][j]), fmaxf(s_m[2][j], s_m[3][j])));
        const float ms = m_new == -INFINITY ? 0.0f : m_new;
        const float corr = __builtin_amdgcn_exp2f(m_run - ms);
        at_s4 ph, pl;
        float psum = 0.0f;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const float p = __builtin_amdgcn_exp2f(sc[r] - ms);
            psum += p;
            ph[r] = bf_bits(p);
            pl[r] = bf_bits(p - bf_val(ph[r]));
        }
        s_p[0][wave][lane] = ph;
        s_p[1][wave][lane] = pl;
        l_run = fmaf(l_run, corr, psum);  // this lane's positions; lane groups and waves are added at the end
        m_run = m_new;
        __syncthreads();
        if (trip > 0) {
#pragma unroll
            for (int i = 0; i < DW; ++i) acc[i] *= corr;
        }
        typedef short s8 __attribute__((ext_vector_type(8)));
        auto join = [](at_s4 x, at_s4 y) { return __builtin_bit_cast(at_b8, (s8){x[0], x[1], x[2], x[3], y[0], y[1], y[2], y[3]}); };
#pragma unroll
        for (int t = 0; t < 4; t += 2) {
            const at_b8 hi = join(s_p[0][t][lane], s_p[0][t + 1][lane]), lw = join(s_p[1][t][lane], s_p[1][t + 1][lane]);
#pragma unroll
            for (int i = 0; i < DW; ++i) {
                const uint8_t* vrow = s_v + (16 * t + 4 * rg + (j >> 2)) * VP + (16 * (wave * DW + i) + 4 * (j & 3)) * 2;
                const at_b8 v = join(lds_tr16(vrow), lds_tr16(vrow + 16 * VP));
                acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, hi, acc[i], 0, 0, 0);
                acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, lw, acc[i], 0, 0, 0);
            }
        }
    }
    l_run += __shfl_xor(l_run, 16, 64);
    l_run += __shfl_xor(l_run, 32, 64);
    if (rg == 0) s_l[wave][j] = l_run;
    __syncthreads();
    if (j >= nh) return;
    const int64_t at = (int64_t)split * a.heads + h0 + j;
    if (wave == 0 && rg == 0) {
        d.pM[at] = m_run * (1.0f / LOG2E);
        d.pL[at] = (s_l[0][j] + s_l[1][j]) + (s_l[2][j] + s_l[3][j]);
    }
#pragma unroll
    for (int i = 0; i < DW; ++i) {
        const int col = 16 * (wave * DW + i) + 4 * rg;
        if (col < a.vdim) *reinterpret_cast<at_f4*>(d.pO + at * a.vdim + col) = acc[i];
    }
}

// grid (heads, ceil(vdim / 64)): out[h][v] = sum over the splits of their results, weighted by exp(m - max) / total.  Four
// waves take every fourth split of 64 values; the results are requested before the weights are known.
__global__ __launch_bounds__(256) void decode_merge_kernel(const float* __restrict__ pO, const float* __restrict__ pM,
                                                           const float* __restrict__ pL, int splits, const ptm_attention_args a,
                                                           float* __restrict__ out) {
    __shared__ float s_sum[4][64];
    const int heads = a.heads, vdim = a.vdim;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, h = blockIdx.x, v = blockIdx.y * 64 + lane, vc = min(v, vdim - 1);
    const float sink = a.sink ? a.sink[h] : -INFINITY, factor = out_factor(a, 0, h, vc);
    float o[16], mv[4], lv[4], m = sink;
#pragma unroll
    for (int u = 0; u < 16; ++u) o[u] = pO[((int64_t)min(wave + 4 * u, splits - 1) * heads + h) * vdim + vc];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
        const int i = min(lane + 64 * u, splits - 1);
        mv[u] = lane + 64 * u < splits ? pM[(int64_t)i * heads + h] : -INFINITY;
        lv[u] = pL[(int64_t)i * heads + h];
        m = fmaxf(m, mv[u]);
    }
    m = max64(m);
    float l = 0.0f;
#pragma unroll
    for (int u = 0; u < 4; ++u) {
        mv[u] = expf(mv[u] - m);  // lane + 64 u: split's weight, 0 past the last
        l = fmaf(lv[u], mv[u], l);
    }
    l = sum64(l);
    if (a.sink) l += expf(sink - m);
    l = factor / l;
    auto weight = [&](int i) {
        const float w = i < 64 ? mv[0] : i < 128 ? mv[1] : i < 192 ? mv[2] : mv[3];  // wave-uniform i
        return __shfl(w, i & 63, 64);
    };
    float acc = 0.0f;
#pragma unroll
    for (int u = 0; u < 16; ++u) acc = fmaf(o[u], weight(wave + 4 * u), acc);
    for (int i = wave + 64; i < splits; i += 4) acc = fmaf(pO[((int64_t)i * heads + h) * vdim + vc], weight(i), acc);
    s_sum[wave][lane] = acc * l;
    __syncthreads();
    if (wave == 0 && v < vdim) out[(int64_t)h * vdim + v] = (s_sum[0][lane] + s_sum[1][lane]) + (s_sum[2][lane] + s_sum[3][lane]);
}

int decode_attention_merge(const float* pO, const float* pM, const float* pL, int splits, const ptm_attention_args& a, float* out,
                           hipStream_t s) {
    if (splits <= 0 || splits > 256) return PTM_E_UNSUPPORTED;
    hipLaunchKernelGGL(decode_merge_kernel, dim3(a.heads, (a.vdim + 63) / 64), dim3(256), 0, s, pO, pM, pL, splits, a, out);
    return launch_status();
}

// tile class of the decode kernel: key size, value size (0: none).  Values that are the keys' first part take them from the
// key rows, so the class's key size covers its value size.
static int decode_class(const ptm_attention_args& a) {
    const int dq = a.dim1 + a.dim2, dv = a.vdim;
    const bool shared = a.V == a.K1 && a.v_row == a.k1_row && a.v_head == a.k1_head && a.dim2 > 0;
    if (dq <= 64 && dv <= 64) return 1;
    if (dq <= 128 && dv <= 64) return 2;
    if (dq <= 128 && dv <= 128) return 3;
    if (dq <= 256 && dv <= 256) return 4;
    if (shared && dq <= 320 && dv <= 256) return 5;
    if (shared && dq <= 576 && dv <= 512) return 6;
    return 0;
}
bool decode_attention_tiled(const ptm_attention_args& a) { return !a.fp32 && decode_class(a) != 0; }

int decode_attention_splits(const ptm_attention_args& a, int max_seq) {
    if (!decode_attention_tiled(a)) return 1;
    const int per = a.heads / a.kv_heads, groups = a.kv_heads * ((per + 15) / 16);
    int chunks = (max_seq + 63) / 64;
    if (a.window > 0) {
        const int w = (a.window + 62) / 64 + 1 + (a.keep_first + 63) / 64;
        chunks = chunks < w ? chunks : w;
    }
    const int cap = groups >= 4 ? 64 : 128;
    return chunks < cap ? chunks : cap;
}

template <int DQ, int DV>
static void decode_launch(const DecodeAttention& d, int splits, dim3 grid, hipStream_t s) {
    const bool shared = d.a.V == d.a.K1 && d.a.dim2 > 0;
    if (d.raw) hipLaunchKernelGGL((decode_mfma_kernel<DQ, DV, true, false>), grid, dim3(256), 0, s, d, splits);
    else if (shared) hipLaunchKernelGGL((decode_mfma_kernel<DQ, DV, false, true>), grid, dim3(256), 0, s, d, splits);
    else hipLaunchKernelGGL((decode_mfma_kernel<DQ, DV, false, false>), grid, dim3(256), 0, s, d, splits);
}

int decode_attention(const DecodeAttention& d, hipStream_t s) {
    const ptm_attention_args& a = d.a;
    const int splits = decode_attention_splits(a, d.max_seq), per = a.heads / a.kv_heads;
    const dim3 grid(splits, a.kv_heads * ((per + 15) / 16));
    switch (decode_class(a)) {
        case 1: decode_launch<64, 64>(d, splits, grid, s); break;
        case 2: decode_launch<128, 64>(d, splits, grid, s); break;
        case 3: decode_launch<128, 128>(d, splits, grid, s); break;
        case 4: decode_launch<256, 256>(d, splits, grid, s); break;
        case 5: hipLaunchKernelGGL((decode_mfma_kernel<320, 256, false, true>), grid, dim3(256), 0, s, d, splits); break;
        case 6: hipLaunchKernelGGL((decode_mfma_kernel<576, 512, false, true>), grid, dim3(256), 0, s, d, splits); break;
        default: return PTM_E_UNSUPPORTED;
    }
    return launch_status();
}

}  // namespace ptm

extern "C" int ptm_attention_rows(const ptm_attention_args* a, ptm_stream_t stream) {
    if (!a) return PTM_E_NULL;
    return ptm::attention_rows(*a, nullptr, false, ptm::as_stream(stream));
}
