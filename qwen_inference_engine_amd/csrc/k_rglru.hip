// k_rglru.hip — the real-gated linear recurrent unit (QIE_MIXER_RGLRU; k_layered.hpp):
//
//   lay::rglru_gates   a = exp(-decay r) and sqrt(1 - a^2) i u of every row and channel, r and i sigmoids of
//                      block-diagonal products of the convolved input u
//   lay::rglru_scan    S = a S + b per channel, times the gelu of the other branch
//   lay::rglru_step    both for steps of few rows, one launch
//
// Everything here is fp32.  The gate products of many rows run on the bf16 matrix cores without losing bits: the
// weights are bf16 already, and u is split into three bf16 parts (8 + 8 + 8 bits, each the truncated rest of the one
// before) whose products with a weight are exact in the fp32 accumulator's inputs; the sum of the three products is the
// fp32 product up to the rounding of its additions.  The bf16 matrix rate is sixteen times the fp32 one, so the three cost
// about a fifth of the one.
#include "k_layered.hpp"

namespace qie {
namespace lay {

namespace {
typedef __bf16 rbf16x8_t __attribute__((ext_vector_type(8)));
typedef float rf32x4_t __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float wsum_r(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
    return v;
}
__device__ __forceinline__ float sigm(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float gelu_t(float z) {
    return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}
// log a = -decay r: a, and what the current input is multiplied by (1 - a^2 without cancellation)
__device__ __forceinline__ void lru_terms(float zr, float zi, float decay, float u, float* a, float* b) {
    const float la = -decay * sigm(zr);
    *a = expf(la);
    *b = sqrtf(-expm1f(2.0f * la)) * sigm(zi) * u;
}
// x as three bf16 words: the top 8 significant bits, the next 8, the last 8
__device__ __forceinline__ void split3(const float* x, uint4* hi, uint4* mid, uint4* lo) {
    uint32_t h[8], m[8], l[8];
#pragma unroll
    for (int i = 0; i < 8; i++) {
        const uint32_t b0 = __float_as_uint(x[i]) & 0xffff0000u;
        const float r1 = x[i] - __uint_as_float(b0);
        const uint32_t b1 = __float_as_uint(r1) & 0xffff0000u;
        const float r2 = r1 - __uint_as_float(b1);
        h[i] = b0 >> 16;
        m[i] = b1 >> 16;
        l[i] = __float_as_uint(r2) >> 16;
    }
    *hi = make_uint4(h[0] | h[1] << 16, h[2] | h[3] << 16, h[4] | h[5] << 16, h[6] | h[7] << 16);
    *mid = make_uint4(m[0] | m[1] << 16, m[2] | m[3] << 16, m[4] | m[5] << 16, m[6] | m[7] << 16);
    *lo = make_uint4(l[0] | l[1] << 16, l[2] | l[3] << 16, l[4] | l[5] << 16, l[6] | l[7] << 16);
}
}  // namespace

// ------------------------------------------------------------------ gates of many rows
// A workgroup takes 128 rows x 16 NC channels of one block, a wave 32 of the rows: D = W u^T, so that a lane ends with four
// neighbouring channels of one row.  Weight fragments (16 channels x 32 inputs) come straight from memory (the four waves
// read the same ones), u fragments are split in registers.
template <int NC>
__global__ __launch_bounds__(256) void rglru_gates_kernel(RgLruP p, int T) {
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, g = lane >> 4, n = lane & 15;
    const int bs = p.bs, per = bs / (16 * NC), blk = blockIdx.x / per, c0 = (blockIdx.x % per) * 16 * NC;
    const int t0 = blockIdx.y * 128 + wave * 32;
    if (t0 >= T) return;
    const uint16_t* wr = (const uint16_t*)p.w + ((int64_t)blk * 2 * bs + c0 + n) * bs + 8 * g;
    const uint16_t* wi = wr + (int64_t)bs * bs;
    const float* ur[2];
#pragma unroll
    for (int m = 0; m < 2; m++) ur[m] = p.u + (int64_t)min(t0 + 16 * m + n, T - 1) * p.ld_u + blk * bs + 8 * g;
    rf32x4_t acc[2][NC][2];   // [gate][channel tile][row tile]
#pragma unroll
    for (int q = 0; q < 2; q++)
#pragma unroll
        for (int c = 0; c < NC; c++)
#pragma unroll
            for (int m = 0; m < 2; m++) acc[q][c][m] = rf32x4_t{0.f, 0.f, 0.f, 0.f};
    float x[2][8];
    auto fetch = [&](int k) {
#pragma unroll
        for (int m = 0; m < 2; m++) {
            *reinterpret_cast<float4*>(x[m]) = *reinterpret_cast<const float4*>(ur[m] + k);
            *reinterpret_cast<float4*>(x[m] + 4) = *reinterpret_cast<const float4*>(ur[m] + k + 4);
        }
    };
    fetch(0);
    for (int k = 0; k < bs; k += 32) {
        uint4 w[2][NC];
#pragma unroll
        for (int c = 0; c < NC; c++) {
            w[0][c] = *reinterpret_cast<const uint4*>(wr + (int64_t)16 * c * bs + k);
            w[1][c] = *reinterpret_cast<const uint4*>(wi + (int64_t)16 * c * bs + k);
        }
        uint4 part[2][3];
#pragma unroll
        for (int m = 0; m < 2; m++) split3(x[m], &part[m][0], &part[m][1], &part[m][2]);
        if (k + 32 < bs) fetch(k + 32);
#pragma unroll
        for (int s = 2; s >= 0; s--)   // the small parts first
#pragma unroll
            for (int m = 0; m < 2; m++)
#pragma unroll
                for (int q = 0; q < 2; q++)
#pragma unroll
                    for (int c = 0; c < NC; c++)
                        acc[q][c][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(rbf16x8_t, w[q][c]),
                                                                               __builtin_bit_cast(rbf16x8_t, part[m][s]), acc[q][c][m], 0, 0, 0);
    }
    const int nch = p.blocks * bs;
#pragma unroll
    for (int c = 0; c < NC; c++) {
        const int ch = blk * bs + c0 + 16 * c + 4 * g;   // four channels of row 16 m + n
        const float4 rb = *reinterpret_cast<const float4*>(p.r_b + ch), ib = *reinterpret_cast<const float4*>(p.i_b + ch);
        const float4 dc = *reinterpret_cast<const float4*>(p.decay + ch);
#pragma unroll
        for (int m = 0; m < 2; m++) {
            const int t = t0 + 16 * m + n;
            if (t >= T) continue;
            const float4 u = *reinterpret_cast<const float4*>(p.u + (int64_t)t * p.ld_u + ch);
            float4 a, b;
            lru_terms(acc[0][c][m][0] + rb.x, acc[1][c][m][0] + ib.x, dc.x, u.x, &a.x, &b.x);
            lru_terms(acc[0][c][m][1] + rb.y, acc[1][c][m][1] + ib.y, dc.y, u.y, &a.y, &b.y);
            lru_terms(acc[0][c][m][2] + rb.z, acc[1][c][m][2] + ib.z, dc.z, u.z, &a.z, &b.z);
            lru_terms(acc[0][c][m][3] + rb.w, acc[1][c][m][3] + ib.w, dc.w, u.w, &a.w, &b.w);
            *reinterpret_cast<float4*>(p.a + (int64_t)t * nch + ch) = a;
            *reinterpret_cast<float4*>(p.b + (int64_t)t * nch + ch) = b;
        }
    }
}

// any other shape, and fp32 weights: the block products by the plain fp32 kernels, then this
__global__ __launch_bounds__(256) void rglru_terms_kernel(RgLruP p, int T) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    const int n = p.blocks * p.bs;
    if (i >= (int64_t)T * n) return;
    const int64_t t = i / n;
    const int c = (int)(i % n), blk = c / p.bs, j = c % p.bs;
    const float* z = p.z + t * 2 * n + (int64_t)blk * 2 * p.bs;
    lru_terms(z[j] + p.r_b[c], z[p.bs + j] + p.i_b[c], p.decay[c], p.u[t * p.ld_u + c], p.a + i, p.b + i);
}

bool rglru_gates_mfma_fits(int bs, bool w_f32) { return !w_f32 && bs % 32 == 0; }

int rglru_gates(const RgLruP& p, int T, hipStream_t st) {
    QIE_REQUIRE(p.u && p.w && p.r_b && p.i_b && p.decay && p.a && p.b && p.blocks > 0 && p.bs > 0 && T > 0, "rglru gates: bad arguments");
    const bool aligned = (((uintptr_t)p.u | (uintptr_t)p.w | (uintptr_t)p.a | (uintptr_t)p.b) & 15) == 0 && p.ld_u % 4 == 0;
    if (rglru_gates_mfma_fits(p.bs, p.w_f32) && aligned) {
        const unsigned rows = (unsigned)((T + 127) / 128);
        if (p.bs % 64 == 0)
            hipLaunchKernelGGL(rglru_gates_kernel<4>, dim3((unsigned)(p.blocks * (p.bs / 64)), rows), dim3(256), 0, st, p, T);
        else
            hipLaunchKernelGGL(rglru_gates_kernel<2>, dim3((unsigned)(p.blocks * (p.bs / 32)), rows), dim3(256), 0, st, p, T);
        QIE_LAUNCH_CHECK();
        return 0;
    }
    QIE_REQUIRE(p.z, "rglru gates: the product scratch is missing");
    const int64_t n = (int64_t)p.blocks * p.bs;
    LinearP l{p.u, p.ld_u, p.w, p.bs, p.z, 2 * n, T, 2 * p.bs, p.bs, p.blocks, p.bs, (int64_t)2 * p.bs * p.bs, 2 * p.bs, 0, nullptr, 0};
    QIE_TRY(linear(l, p.w_f32 != 0, st));
    hipLaunchKernelGGL(rglru_terms_kernel, dim3((unsigned)((T * n + 255) / 256)), dim3(256), 0, st, p, T);
    QIE_LAUNCH_CHECK();
    return 0;
}

// ------------------------------------------------------------------ recurrence
// One thread per (entry, channel); the loads of the next rows do not depend on the recurrence and run ahead of it.
__global__ __launch_bounds__(64) void rglru_scan_kernel(RgLruP p) {
    const int n = p.blocks * p.bs, c = blockIdx.x * 64 + threadIdx.x;
    if (c >= n) return;
    const int4 en = p.entries[blockIdx.y];   // {first packed row, rows, index, first position}
    float S = 0.f, run = 1.f;
    if (p.init && (!p.init_if_pos || en.w > 0)) S = p.init[(int64_t)en.z * p.init_stride + p.init_off + c];
    const bool outs = p.want_out != 0;
    const float yb = outs ? p.y_b[c] : 0.f;
    constexpr int U = 8;
    for (int t0 = 0; t0 < en.y; t0 += U) {
        float ra[U], rb[U], ry[U];
#pragma unroll
        for (int k = 0; k < U; k++) {
            const int64_t t = en.x + (t0 + k < en.y ? t0 + k : t0);
            ra[k] = p.a[t * n + c];
            rb[k] = p.b[t * n + c];
            ry[k] = outs ? p.y[t * p.ld_y + c] : 0.f;
        }
#pragma unroll
        for (int k = 0; k < U; k++) {
            if (t0 + k >= en.y) break;
            S = fmaf(ra[k], S, rb[k]);
            run *= ra[k];
            if (outs) {
                const float o = S * gelu_t(ry[k] + yb);
                const int64_t oi = (int64_t)(en.x + t0 + k) * p.ld_out + c;
                if (p.out) p.out[oi] = o;
                if (p.out_bf) p.out_bf[oi] = f2bf(o);
            }
        }
    }
    if (p.end) p.end[(int64_t)en.z * p.end_stride + p.end_off + c] = S;
    if (p.decay_out) p.decay_out[(int64_t)en.z * p.end_stride + p.end_off + c] = run;
}

int rglru_scan(const RgLruP& p, hipStream_t st) {
    QIE_REQUIRE(p.a && p.b && p.entries && p.n_entries > 0 && (!p.want_out || (p.y && p.y_b && (p.out || p.out_bf))) && (p.want_out || p.end),
                "rglru scan: bad arguments");
    const int n = p.blocks * p.bs;
    hipLaunchKernelGGL(rglru_scan_kernel, dim3((unsigned)((n + 63) / 64), (unsigned)p.n_entries), dim3(64), 0, st, p);
    QIE_LAUNCH_CHECK();
    return 0;
}

// ------------------------------------------------------------------ steps of few rows
// A wave per channel: its two weight rows against every row's block of u, eight rows a turn; lane t then owns row t (gates,
// the other branch, the slot's state: all rows' loads and exponentials at once), and rows of one entry, neighbours at most
// `chain` long, hand their state to the next lane.  V inputs per lane and load.
template <typename TW, int V> __device__ __forceinline__ void ldw_r(const TW* p, float* o) {
    if constexpr (V == 1) {
        if constexpr (sizeof(TW) == 4) o[0] = p[0];
        else o[0] = bf2f(p[0]);
    } else if constexpr (sizeof(TW) == 4) {
        *reinterpret_cast<float4*>(o) = *reinterpret_cast<const float4*>(p);
    } else {
        const uint2 u = *reinterpret_cast<const uint2*>(p);
        o[0] = bf2f(u.x & 0xffffu); o[1] = bf2f(u.x >> 16); o[2] = bf2f(u.y & 0xffffu); o[3] = bf2f(u.y >> 16);
    }
}

template <typename TW, int V>
__global__ __launch_bounds__(256) void rglru_step_kernel(RgLruP p, int T, int chain) {
    const int n = p.blocks * p.bs, bs = p.bs, lane = threadIdx.x & 63, c = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (c >= n) return;
    const int blk = c / bs, j = c % bs;
    const TW* wr = (const TW*)p.w + ((int64_t)blk * 2 * bs + j) * bs;
    const TW* wi = wr + (int64_t)bs * bs;
    // this lane's row
    const int row = min(lane, T - 1);
    const int64_t so = (int64_t)p.row_slot[row] * p.init_stride + p.init_off + c;
    const int k = p.row_k[row];
    const bool last = row + 1 == T || p.row_k[min(row + 1, T - 1)] == 0;
    float S = k == 0 && p.row_pos[row] > 0 ? p.init[so] : 0.f;
    const float uc = p.u[row * p.ld_u + c], yc = p.y[row * p.ld_y + c] + p.y_b[c];
    float zr = p.r_b[c], zi = p.i_b[c];
    constexpr int R = 8;
    for (int t0 = 0; t0 < T; t0 += R) {
        float ar[R], ai[R];
        const float* ub[R];
#pragma unroll
        for (int r = 0; r < R; r++) {
            ub[r] = p.u + (int64_t)min(t0 + r, T - 1) * p.ld_u + blk * bs;
            ar[r] = ai[r] = 0.f;
        }
        for (int q = lane * V; q < bs; q += 64 * V) {
            float a[V], b[V], x[R][V];
            ldw_r<TW, V>(wr + q, a);
            ldw_r<TW, V>(wi + q, b);
#pragma unroll
            for (int r = 0; r < R; r++) ldw_r<float, V>(ub[r] + q, x[r]);
#pragma unroll
            for (int r = 0; r < R; r++)
#pragma unroll
                for (int v = 0; v < V; v++) {
                    ar[r] = fmaf(a[v], x[r][v], ar[r]);
                    ai[r] = fmaf(b[v], x[r][v], ai[r]);
                }
        }
#pragma unroll
        for (int r = 0; r < R; r++) {
            const float sr = wsum_r(ar[r]), si = wsum_r(ai[r]);
            if (lane == t0 + r) {
                zr += sr;
                zi += si;
            }
        }
    }
    float a, b;
    lru_terms(zr, zi, p.decay[c], uc, &a, &b);
    if (k == 0) S = fmaf(a, S, b);
    for (int s = 1; s < chain; s++) {
        const float prev = __shfl_up(S, 1, 64);
        if (k == s) S = fmaf(a, prev, b);
    }
    if (lane >= T) return;
    const float o = S * gelu_t(yc);
    if (p.out) p.out[(int64_t)row * p.ld_out + c] = o;
    if (p.out_bf) p.out_bf[(int64_t)row * p.ld_out + c] = f2bf(o);
    if (last) p.end[so] = S;
}

int rglru_step(const RgLruP& p, int T, int chain, hipStream_t st) {
    QIE_REQUIRE(p.u && p.w && p.y && p.y_b && p.row_slot && p.row_pos && p.row_k && p.init && p.end && (p.out || p.out_bf) && T > 0 &&
                    T <= kRgLruStepRows && chain >= 1 && p.init == p.end && p.init_stride == p.end_stride && p.init_off == p.end_off,
                "rglru step: bad arguments");
    const dim3 grid((unsigned)((p.blocks * p.bs + 3) / 4));
    const bool v4 = p.bs % 4 == 0 && p.ld_u % 4 == 0 && (((uintptr_t)p.u | (uintptr_t)p.w) & 15) == 0;
    if (p.w_f32 && v4)
        hipLaunchKernelGGL((rglru_step_kernel<float, 4>), grid, dim3(256), 0, st, p, T, chain);
    else if (p.w_f32)
        hipLaunchKernelGGL((rglru_step_kernel<float, 1>), grid, dim3(256), 0, st, p, T, chain);
    else if (v4)
        hipLaunchKernelGGL((rglru_step_kernel<uint16_t, 4>), grid, dim3(256), 0, st, p, T, chain);
    else
        hipLaunchKernelGGL((rglru_step_kernel<uint16_t, 1>), grid, dim3(256), 0, st, p, T, chain);
    QIE_LAUNCH_CHECK();
    return 0;
}

}  // namespace lay
}  // namespace qie
