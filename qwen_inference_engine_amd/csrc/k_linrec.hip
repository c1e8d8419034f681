// k_linrec.hip — decayed linear recurrences of the layered engine tier (k_layered.hpp):
//
//   lay::linrec_step      rows in order on the vector units (entries of few rows)
//   lay::linrec_walk      16 rows at a time on the fp32 matrix cores, the state in registers
//   lay::linrec_carry     states that enter the pieces of long entries
//   lay::low_rank_log_sigmoid   second stage of a low-rank decay projection, as a log decay
//
// One state form S [dim][vdim] per head, S = diag(a) S + m k v^T, o = S^T q, serves the gated linear
// attention (a per key channel) and the state space (one a per head, its step size on k, a skip on v).
// Everything here is fp32, matrix products included (v_mfma_f32_16x16x4_f32).
#include "k_layered.hpp"

namespace qie {
namespace lay {

namespace {

typedef float f32x4_t __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float softplus(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

}  // namespace

// One value of the low-rank log decay (LinRecP.lr_in)
__device__ __forceinline__ float low_rank_log(const LinRecP& p, int64_t t, int c) {
    const float* a = p.lr_in + t * p.ld_lr;
    float z = 0.f;
    if (p.lr_w_f32) {
        const float* w = (const float*)p.lr_w + (int64_t)c * p.rank;
        for (int r = 0; r < p.rank; r++) z = fmaf(w[r], a[r], z);
    } else {
        const uint16_t* w = (const uint16_t*)p.lr_w + (int64_t)c * p.rank;
        int r = 0;
        if ((p.rank & 7) == 0)
#pragma unroll 2
            for (; r < p.rank; r += 8) {
                const uint4 u = *reinterpret_cast<const uint4*>(w + r);
                z = fmaf(bf2f(u.x & 0xffffu), a[r], z);
                z = fmaf(bf2f(u.x >> 16), a[r + 1], z);
                z = fmaf(bf2f(u.y & 0xffffu), a[r + 2], z);
                z = fmaf(bf2f(u.y >> 16), a[r + 3], z);
                z = fmaf(bf2f(u.z & 0xffffu), a[r + 4], z);
                z = fmaf(bf2f(u.z >> 16), a[r + 5], z);
                z = fmaf(bf2f(u.w & 0xffffu), a[r + 6], z);
                z = fmaf(bf2f(u.w >> 16), a[r + 7], z);
            }
        for (; r < p.rank; r++) z = fmaf(bf2f(w[r]), a[r], z);
    }
    return -softplus(-(z + p.lr_bias[c])) * p.inv_tau;
}

// ------------------------------------------------------------------ rows in order
// One block per (head, entry, 64 value columns); a thread owns SR state rows of one column, blockDim / 64 thread
// groups split dim.  TT rows a turn: their q, k and decays staged in LDS, the groups' partial outputs summed there.
template <int SR>
__global__ __launch_bounds__(1024) void linrec_step_kernel(LinRecP p, int dimP) {
    constexpr int TT = 4;
    extern __shared__ __align__(16) float sm[];
    const int NG = blockDim.x >> 6;
    float* qs = sm;                 // [TT][dimP]
    float* ks = qs + TT * dimP;     // [TT][dimP], step size applied
    float* as = ks + TT * dimP;     // [TT][dimP]
    float* op = as + TT * dimP;     // [TT][NG][64]
    const int h = blockIdx.x, c0 = blockIdx.z * 64, tid = threadIdx.x, lane = tid & 63, grp = tid >> 6;
    const int4 en = p.entries[blockIdx.y];
    const int dim = p.dim, vdim = p.vdim, c = c0 + lane, d0 = grp * SR;
    const bool cok = c < vdim;
    const int64_t so = (int64_t)h * dim * vdim;
    const bool warm = p.init && (!p.init_if_pos || en.w > 0);
    const float* st0 = p.init + (int64_t)en.z * p.init_stride + p.init_off + so;
    float S[SR];
#pragma unroll
    for (int r = 0; r < SR; r++) S[r] = (warm && cok && d0 + r < dim) ? st0[(int64_t)(d0 + r) * vdim + c] : 0.f;
    const float ah = p.dt ? p.a_h[h] : 0.f, db = p.dt ? p.dt_bias[h] : 0.f, skip = p.skip ? p.skip[h] : 0.f;
    const int64_t qk0 = (int64_t)(h / p.rep) * dim, HV = (int64_t)p.heads * vdim;
    for (int t0 = 0; t0 < en.y; t0 += TT) {
        const int nt = min(TT, en.y - t0);
        float v[TT];
#pragma unroll
        for (int tt = 0; tt < TT; tt++) v[tt] = (tt < nt && cok) ? p.v[(int64_t)(en.x + t0 + tt) * p.ldv + (int64_t)h * vdim + c] : 0.f;
        __syncthreads();   // the previous turn's readers are done
        for (int i = tid; i < nt * dimP; i += blockDim.x) {
            const int tt = i / dimP, d = i % dimP;
            const int64_t t = en.x + t0 + tt;
            float q = 0.f, k = 0.f, a = 1.f;
            if (d < dim) {
                q = p.q[t * p.ldq + qk0 + d] * p.q_scale;
                k = p.k[t * p.ldk + qk0 + d];
                if (p.dt) {
                    const float dt = softplus(p.dt[t * p.ld_dt + h] + db);
                    a = expf(-ah * dt);
                    k *= dt;
                } else if (p.log_decay) {
                    a = expf(p.log_decay[t * p.heads * dim + (int64_t)h * dim + d]);
                } else {
                    a = expf(low_rank_log(p, t, h * dim + d));
                }
            }
            qs[i] = q;
            ks[i] = k;
            as[i] = a;
        }
        __syncthreads();
#pragma unroll
        for (int tt = 0; tt < TT; tt++) {
            if (tt < nt) {
                float o = 0.f;
                const float *qt = qs + tt * dimP + d0, *kt = ks + tt * dimP + d0, *at = as + tt * dimP + d0;
#pragma unroll
                for (int r = 0; r < SR; r++) {
                    S[r] = fmaf(at[r], S[r], kt[r] * v[tt]);
                    o = fmaf(S[r], qt[r], o);
                }
                op[(tt * NG + grp) * 64 + lane] = o;
            }
        }
        __syncthreads();
        for (int i = tid; i < nt * 64; i += blockDim.x) {
            const int tt = i >> 6, cl = i & 63;
            float o = 0.f;
            for (int g = 0; g < NG; g++) o += op[(tt * NG + g) * 64 + cl];
            if (c0 + cl < vdim) {
                const int64_t t = en.x + t0 + tt;
                if (p.skip) o = fmaf(skip, p.v[t * p.ldv + (int64_t)h * vdim + c0 + cl], o);
                p.out[t * HV + (int64_t)h * vdim + c0 + cl] = o;
            }
        }
    }
    if (!p.end) return;
    float* st1 = p.end + (int64_t)en.z * p.end_stride + p.end_off + so;
#pragma unroll
    for (int r = 0; r < SR; r++)
        if (cok && d0 + r < dim) st1[(int64_t)(d0 + r) * vdim + c] = S[r];
}

static int linrec_check(const LinRecP& p) {
    QIE_REQUIRE(p.q && p.k && p.v && p.entries && p.n_entries > 0 && p.heads > 0 && p.dim > 0 && p.vdim > 0 && p.rep > 0 &&
                    p.heads % p.rep == 0 && (p.log_decay != nullptr) + (p.dt != nullptr) + (p.lr_in != nullptr) == 1 &&
                    (!p.dt || (p.dt_bias && p.a_h)) && (!p.lr_in || (p.lr_w && p.lr_bias && p.rank > 0)),
                "linear recurrence: bad arguments");
    return 0;
}

int linrec_step(const LinRecP& p, hipStream_t st) {
    QIE_TRY(linrec_check(p));
    QIE_REQUIRE(p.dim <= 512 && p.out && !p.decay, "linear recurrence: rows in order take dim up to 512 (%d)", p.dim);
    const int SR = p.dim <= 128 ? 8 : 32, NG = (p.dim + SR - 1) / SR, dimP = NG * SR;
    const size_t shm = (size_t)4 * (3 * dimP + NG * 64) * 4;
    dim3 grid((unsigned)p.heads, (unsigned)p.n_entries, (unsigned)((p.vdim + 63) / 64));
    if (SR == 8)
        hipLaunchKernelGGL(linrec_step_kernel<8>, grid, dim3(64 * NG), shm, st, p, dimP);
    else
        hipLaunchKernelGGL(linrec_step_kernel<32>, grid, dim3(64 * NG), shm, st, p, dimP);
    QIE_LAUNCH_CHECK();
    return 0;
}

// ------------------------------------------------------------------ 16 rows at a time on the matrix cores
// One block per (head, entry, 64 value columns), a wave per 16 columns.  With L_t the sum of the tile's log decays up
// to row t and L the whole tile's: o_t = (q_t e^(L_t)) S + sum_(s <= t) P_ts v_s, P_ts = sum_d q_td k_sd e^(L_t - L_s),
// S <- e^L S + sum_s (k_s e^(L - L_s)) v_s^T.  All three are products of 16 x 16 x 4 fp32 tiles.  The accumulator
// layout of S (register i of lane group g = row 4g + i of a tile) is a B operand as it stands when k-slot g of the
// i-th product stands for row 4g + i, so the state never leaves the registers; P is made transposed, which is the
// A operand of the second product in the same way.
//
// A stage brings two 16-row tiles to LDS (the next stage's rows in registers meanwhile); the four waves make the two
// P tiles (two halves of dim each), then walk both tiles for their own columns.
//
// Decay per key channel: q e^(L_t) and k e^(L - L_s) (both at most the value itself) are what LDS holds; P takes
// e^(-L) on its q side, exact as long as every |L| of the stage stays below kSpan (e^kSpan is far inside fp32).  A
// stage that decays faster computes P pair by pair from the unscaled values.  Decay per head: L is one number per
// row, so P is scaled after the product and nothing can overflow.
constexpr int kStage = 32;
constexpr float kSpan = 40.f;

template <int DT, bool SCALAR>
__global__ __launch_bounds__(256) void linrec_walk_kernel(LinRecP p, int vec) {
    constexpr int dimP = 16 * DT, LQ = dimP + 4, LV = 68, LP = 20, NI = (2 * dimP + 255) / 256;
    __shared__ __align__(16) float qs[kStage * LQ];
    __shared__ __align__(16) float ks[kStage * LQ];
    __shared__ __align__(16) float vs[kStage * LV];
    __shared__ __align__(16) float ps[2][2][16 * LP];              // [half of dim][tile][t][s]
    __shared__ __align__(16) float wt[SCALAR ? 4 : 2 * dimP];      // key decay: e^(-L) per tile and channel
    __shared__ __align__(16) float et[SCALAR ? 4 : 2 * dimP];      // e^L per tile (and channel)
    __shared__ float sL[SCALAR ? kStage : 1], sdt[SCALAR ? kStage : 1], eL[SCALAR ? kStage : 1], kf[SCALAR ? kStage : 1];
    // neighbouring blocks go to different dies: heads that share q and k rows sit 8 blocks apart, on one die's cache
    const int h = p.heads % 8 == 0 ? (int)(blockIdx.x % 8) * (p.heads / 8) + (int)(blockIdx.x / 8) : (int)blockIdx.x;
    const int c0 = blockIdx.z * 64, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, g = lane >> 4, n = lane & 15;
    const int4 en = p.entries[blockIdx.y];
    const int dim = p.dim, vdim = p.vdim, col = c0 + wave * 16 + n;
    const bool cok = col < vdim, outs = p.out != nullptr;
    const int64_t so = (int64_t)h * dim * vdim, qk0 = (int64_t)(h / p.rep) * dim, HV = (int64_t)p.heads * vdim;
    const float ah = SCALAR ? p.a_h[h] : 0.f, db = SCALAR ? p.dt_bias[h] : 0.f, skip = p.skip ? p.skip[h] : 0.f;
    f32x4_t S[DT];
    {
        const bool warm = p.init && (!p.init_if_pos || en.w > 0) && cok;
        const float* st0 = p.init + (int64_t)en.z * p.init_stride + p.init_off + so;
#pragma unroll
        for (int j = 0; j < DT; j++)
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int d = 16 * j + 4 * g + i;
                S[j][i] = (warm && d < dim) ? st0[(int64_t)d * vdim + col] : 0.f;
            }
    }
    // the rows of a stage.  Decay per channel: a thread owns channel d of tile x (column i = x * dimP + d) of q, k and the
    // decays; at up to 64 channels the block's upper half takes k (and needs the decays as well), the lower half q.
    // Decay per head: q and k come as they lie, four channels of a row per load.
    constexpr int NK = (8 * dimP + 255) / 256, D4 = dimP / 4;
    constexpr bool TWO = DT <= 4;
    const int ctid = TWO ? tid & 127 : tid;
    const bool do_q = !TWO || tid < 128, do_k = !TWO || tid >= 128;
    float rq[SCALAR ? 1 : NI][16], rk[SCALAR ? 1 : NI][16], rl[SCALAR ? 1 : NI][16], rdt = 0.f, run[SCALAR ? 1 : NI] = {};
    float4 fq[SCALAR ? NK : 1], fk[SCALAR ? NK : 1], rv[2];
    auto four = [&](const float* base, int64_t at, int c, int lim, bool ok) -> float4 {
        float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
        if (!ok || c >= lim) return o;
        if (vec) return *reinterpret_cast<const float4*>(base + at + c);
        o.x = base[at + c];
        if (c + 1 < lim) o.y = base[at + c + 1];
        if (c + 2 < lim) o.z = base[at + c + 2];
        if (c + 3 < lim) o.w = base[at + c + 3];
        return o;
    };
    auto fetch = [&](int t0) {
        if (SCALAR) {
#pragma unroll
            for (int k = 0; k < NK; k++) {
                const int i = tid + 256 * k, tt = t0 + i / D4, d = i % D4 * 4;
                const bool ok = i < kStage * D4 && tt < en.y;
                const int64_t t = en.x + (ok ? tt : 0);
                if (outs) fq[k] = four(p.q, t * p.ldq + qk0, d, dim, ok);
                fk[k] = four(p.k, t * p.ldk + qk0, d, dim, ok);
            }
        } else {
#pragma unroll
            for (int k = 0; k < NI; k++) {
                const int i = ctid + 256 * k, x = i / dimP, d = i % dimP;
                const bool on = i < 2 * dimP && d < dim;
#pragma unroll
                for (int r = 0; r < 16; r++) {
                    const int tt = t0 + 16 * x + r;
                    const bool ok = on && tt < en.y;
                    const int64_t t = en.x + (ok ? tt : 0);
                    if (outs && do_q) rq[k][r] = ok ? p.q[t * p.ldq + qk0 + d] : 0.f;
                    if (do_k) rk[k][r] = ok ? p.k[t * p.ldk + qk0 + d] : 0.f;
                    rl[k][r] = ok ? p.log_decay[t * p.heads * dim + (int64_t)h * dim + d] : 0.f;
                }
            }
        }
#pragma unroll
        for (int k = 0; k < 2; k++) {
            const int tt = t0 + (tid >> 4) + 16 * k;
            rv[k] = four(p.v, (int64_t)(en.x + tt) * p.ldv + (int64_t)h * vdim, c0 + (tid & 15) * 4, vdim, tt < en.y);
        }
        if (SCALAR && tid < kStage) rdt = t0 + tid < en.y ? p.dt[(int64_t)(en.x + t0 + tid) * p.ld_dt + h] : 0.f;
    };
    fetch(0);
    for (int t0 = 0; t0 < en.y; t0 += kStage) {
        __syncthreads();   // the previous stage has been read
        int steep = 0;
#pragma unroll
        for (int k = 0; k < 2; k++) *reinterpret_cast<float4*>(vs + ((tid >> 4) + 16 * k) * LV + (tid & 15) * 4) = rv[k];
        if (SCALAR) {
#pragma unroll
            for (int k = 0; k < NK; k++) {
                const int i = tid + 256 * k, at = i / D4 * LQ + i % D4 * 4;
                if (i < kStage * D4) {
                    if (outs)
                        *reinterpret_cast<float4*>(qs + at) = make_float4(fq[k].x * p.q_scale, fq[k].y * p.q_scale, fq[k].z * p.q_scale,
                                                                          fq[k].w * p.q_scale);
                    *reinterpret_cast<float4*>(ks + at) = fk[k];
                }
            }
            if (tid < kStage) {
                const float dt = t0 + tid < en.y ? softplus(rdt + db) : 0.f;
                float L = -ah * dt;
#pragma unroll
                for (int o = 1; o < 16; o <<= 1) {
                    const float up = __shfl_up(L, o, 16);
                    if ((tid & 15) >= o) L += up;
                }
                const float tot = __shfl(L, 15, 16);
                sL[tid] = L;
                sdt[tid] = dt;
                eL[tid] = __expf(L);
                kf[tid] = dt * __expf(tot - L);
                if ((tid & 15) == 15) et[tid >> 4] = __expf(tot);
                run[0] += tot;
            }
            __syncthreads();
        } else {
#pragma unroll
            for (int k = 0; k < NI; k++) {
                const int i = ctid + 256 * k;
#pragma unroll
                for (int r = 1; r < 16; r++) rl[k][r] += rl[k][r - 1];
                if (i < 2 * dimP) {
                    et[i] = __expf(rl[k][15]);
                    wt[i] = __expf(fminf(-rl[k][15], kSpan));
                    run[k] += rl[k][15];
                    steep |= rl[k][15] < -kSpan;
                }
            }
            if (outs && __syncthreads_or(steep)) {
                steep = 1;
                for (int x = 0; x < 2; x++) {      // P pair by pair: unscaled q and k, and L, of one tile at a time
#pragma unroll
                    for (int k = 0; k < NI; k++) {
                        const int i = ctid + 256 * k, d = i % dimP;
                        if (i < 2 * dimP && i / dimP == x)
#pragma unroll
                            for (int r = 0; r < 16; r++) {
                                if (do_q) qs[r * LQ + d] = rq[k][r] * p.q_scale;
                                if (do_k) ks[r * LQ + d] = rk[k][r];
                                if (do_q) qs[(16 + r) * LQ + d] = rl[k][r];
                            }
                    }
                    __syncthreads();
                    const int t = tid & 15, s = tid >> 4;
                    float a = 0.f;
                    if (s <= t)
                        for (int d = 0; d < dim; d++)
                            a = fmaf(qs[t * LQ + d] * ks[s * LQ + d], __expf(qs[(16 + t) * LQ + d] - qs[(16 + s) * LQ + d]), a);
                    ps[0][x][t * LP + s] = a;
                    ps[1][x][t * LP + s] = 0.f;
                    __syncthreads();
                }
            }
#pragma unroll
            for (int k = 0; k < NI; k++) {
                const int i = ctid + 256 * k, x = i / dimP, d = i % dimP;
                if (i < 2 * dimP)
#pragma unroll
                    for (int r = 0; r < 16; r++) {
                        if (outs && do_q) qs[(16 * x + r) * LQ + d] = rq[k][r] * p.q_scale * __expf(rl[k][r]);
                        if (do_k) ks[(16 * x + r) * LQ + d] = rk[k][r] * __expf(rl[k][15] - rl[k][r]);
                    }
            }
            __syncthreads();
        }
        if (t0 + kStage < en.y) fetch(t0 + kStage);
        if (outs && (SCALAR || !steep)) {
            // P^T of tile x over one half of dim: A = k rows, B = q rows
            const int x = wave & 1, half = wave >> 1;
            constexpr int J0 = (DT + 1) / 2;
            f32x4_t a = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int jj = 0; jj < J0; jj++) {
                const int j = half * J0 + jj;
                if (j < DT) {
                    const float4 kk = *reinterpret_cast<const float4*>(ks + (16 * x + n) * LQ + 16 * j + 4 * g);
                    float4 qq = *reinterpret_cast<const float4*>(qs + (16 * x + n) * LQ + 16 * j + 4 * g);
                    if (!SCALAR) {
                        const float4 w = *reinterpret_cast<const float4*>(wt + x * dimP + 16 * j + 4 * g);
                        qq.x *= w.x;
                        qq.y *= w.y;
                        qq.z *= w.z;
                        qq.w *= w.w;
                    }
                    a = __builtin_amdgcn_mfma_f32_16x16x4f32(kk.x, qq.x, a, 0, 0, 0);
                    a = __builtin_amdgcn_mfma_f32_16x16x4f32(kk.y, qq.y, a, 0, 0, 0);
                    a = __builtin_amdgcn_mfma_f32_16x16x4f32(kk.z, qq.z, a, 0, 0, 0);
                    a = __builtin_amdgcn_mfma_f32_16x16x4f32(kk.w, qq.w, a, 0, 0, 0);
                }
            }
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int s = 4 * g + i;
                float v = s <= n ? a[i] : 0.f;
                if (SCALAR) v = s <= n ? v * (sdt[16 * x + s] * __expf(sL[16 * x + n] - sL[16 * x + s])) : 0.f;
                a[i] = v;
            }
            *reinterpret_cast<float4*>(&ps[half][x][n * LP + 4 * g]) = make_float4(a[0], a[1], a[2], a[3]);
        }
        if (outs) __syncthreads();
#pragma unroll
        for (int x = 0; x < 2; x++) {
            if (t0 + 16 * x >= en.y) break;
            float vb[4];
#pragma unroll
            for (int i = 0; i < 4; i++) vb[i] = vs[(16 * x + 4 * g + i) * LV + wave * 16 + n];
            if (outs) {
                f32x4_t a0 = {0.f, 0.f, 0.f, 0.f}, a1 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int j = 0; j < DT; j++) {
                    const float4 qq = *reinterpret_cast<const float4*>(qs + (16 * x + n) * LQ + 16 * j + 4 * g);
                    a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(qq.x, S[j][0], a0, 0, 0, 0);
                    a1 = __builtin_amdgcn_mfma_f32_16x16x4f32(qq.y, S[j][1], a1, 0, 0, 0);
                    a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(qq.z, S[j][2], a0, 0, 0, 0);
                    a1 = __builtin_amdgcn_mfma_f32_16x16x4f32(qq.w, S[j][3], a1, 0, 0, 0);
                }
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    a0[i] += a1[i];
                    if (SCALAR) a0[i] *= eL[16 * x + 4 * g + i];
                }
                const float4 p0 = *reinterpret_cast<const float4*>(&ps[0][x][n * LP + 4 * g]);
                const float4 p1 = *reinterpret_cast<const float4*>(&ps[1][x][n * LP + 4 * g]);
                a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(p0.x + p1.x, vb[0], a0, 0, 0, 0);
                a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(p0.y + p1.y, vb[1], a0, 0, 0, 0);
                a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(p0.z + p1.z, vb[2], a0, 0, 0, 0);
                a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(p0.w + p1.w, vb[3], a0, 0, 0, 0);
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    const int tt = t0 + 16 * x + 4 * g + i;
                    if (cok && tt < en.y) p.out[(int64_t)(en.x + tt) * HV + (int64_t)h * vdim + col] = fmaf(skip, vb[i], a0[i]);
                }
            }
            if (SCALAR) {
                const float e = et[x];
#pragma unroll
                for (int i = 0; i < 4; i++) vb[i] *= kf[16 * x + 4 * g + i];
#pragma unroll
                for (int j = 0; j < DT; j++)
#pragma unroll
                    for (int i = 0; i < 4; i++) S[j][i] *= e;
            } else {
#pragma unroll
                for (int j = 0; j < DT; j++) {
                    const float4 e = *reinterpret_cast<const float4*>(et + x * dimP + 16 * j + 4 * g);
                    S[j][0] *= e.x;
                    S[j][1] *= e.y;
                    S[j][2] *= e.z;
                    S[j][3] *= e.w;
                }
            }
#pragma unroll
            for (int i = 0; i < 4; i++)   // the tiles' products are independent, a tile's four are not
#pragma unroll
                for (int j = 0; j < DT; j++)
                    S[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(ks[(16 * x + 4 * g + i) * LQ + 16 * j + n], vb[i], S[j], 0, 0, 0);
        }
    }
    if (p.end && cok) {
        float* st1 = p.end + (int64_t)en.z * p.end_stride + p.end_off + so;
#pragma unroll
        for (int j = 0; j < DT; j++)
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int d = 16 * j + 4 * g + i;
                if (d < dim) st1[(int64_t)d * vdim + col] = S[j][i];
            }
    }
    if (p.decay && blockIdx.z == 0) {
        // the entry's whole log decay: the two tile columns of a channel meet in LDS
        float* dec = p.decay + ((int64_t)blockIdx.y * p.heads + h) * dim;
        __syncthreads();
        if (SCALAR) {
            if (tid < kStage && (tid & 15) == 0) et[tid >> 4] = run[0];
            __syncthreads();
            for (int d = tid; d < dim; d += 256) dec[d] = __expf(et[0] + et[1]);
        } else {
#pragma unroll
            for (int k = 0; k < NI; k++) {
                const int i = ctid + 256 * k;
                if (i < 2 * dimP) et[i] = run[k];
            }
            __syncthreads();
            for (int d = tid; d < dim; d += 256) dec[d] = __expf(et[d] + et[dimP + d]);
        }
    }
}

bool linrec_walk_fits(int dim, int vdim) { return dim >= 1 && dim <= 256 && vdim >= 1; }

template <int DT>
static void linrec_walk_launch(const LinRecP& p, dim3 grid, hipStream_t st) {
    auto rows16 = [](const float* b, int64_t ld) { return ((uintptr_t)b & 15) == 0 && ld % 4 == 0; };
    const int vec = rows16(p.q, p.ldq) && rows16(p.k, p.ldk) && rows16(p.v, p.ldv) && p.dim % 4 == 0 && p.vdim % 4 == 0;
    if (p.dt)
        hipLaunchKernelGGL((linrec_walk_kernel<DT, true>), grid, dim3(256), 0, st, p, vec);
    else
        hipLaunchKernelGGL((linrec_walk_kernel<DT, false>), grid, dim3(256), 0, st, p, vec);
}

int linrec_walk(const LinRecP& p, hipStream_t st) {
    QIE_TRY(linrec_check(p));
    QIE_REQUIRE(!p.lr_in && linrec_walk_fits(p.dim, p.vdim), "linear recurrence: dim %d above the matrix-core form's 256", p.dim);
    dim3 grid((unsigned)p.heads, (unsigned)p.n_entries, (unsigned)((p.vdim + 63) / 64));
    const int dt = (p.dim + 15) / 16;
    if (dt <= 1) linrec_walk_launch<1>(p, grid, st);
    else if (dt <= 2) linrec_walk_launch<2>(p, grid, st);
    else if (dt <= 4) linrec_walk_launch<4>(p, grid, st);
    else if (dt <= 8) linrec_walk_launch<8>(p, grid, st);
    else linrec_walk_launch<16>(p, grid, st);
    QIE_LAUNCH_CHECK();
    return 0;
}

// ------------------------------------------------------------------ states entering the pieces
// One thread per state element; the next piece's loads are in flight while this one's state is stored.
__global__ __launch_bounds__(256) void linrec_carry_kernel(LinRecCarryP p) {
    const int64_t n = (int64_t)p.heads * p.dim * p.vdim, HD = (int64_t)p.heads * p.dim;
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    const int4 sp = p.spans[blockIdx.y];
    const int64_t hd = i / p.vdim;
    float* stp = p.state + (int64_t)sp.z * p.slot_stride + p.state_off + i;
    float S = sp.w > 0 ? *stp : 0.f;
    float nd = p.decay[(int64_t)sp.x * HD + hd], nl = p.s_loc[(int64_t)sp.x * n + i];
    for (int c = sp.x; c < sp.x + sp.y; c++) {
        const float d = nd, l = nl;
        const int cn = min(c + 1, sp.x + sp.y - 1);
        nd = p.decay[(int64_t)cn * HD + hd];
        nl = p.s_loc[(int64_t)cn * n + i];
        p.s_in[(int64_t)c * n + i] = S;
        S = fmaf(d, S, l);
    }
    *stp = S;
}
int linrec_carry(const LinRecCarryP& p, hipStream_t st) {
    QIE_REQUIRE(p.n_spans > 0 && p.s_loc && p.decay && p.s_in && p.state, "linear recurrence carry: bad arguments");
    const int64_t n = (int64_t)p.heads * p.dim * p.vdim;
    hipLaunchKernelGGL(linrec_carry_kernel, dim3((unsigned)((n + 255) / 256), (unsigned)p.n_spans), dim3(256), 0, st, p);
    QIE_LAUNCH_CHECK();
    return 0;
}

// ------------------------------------------------------------------ low-rank log decays
// One block per (256 channels, LR rows): the rows' first-stage values in LDS, a channel's weight row streamed once.
constexpr int LR = 8;

template <typename TW> __device__ __forceinline__ float ldw(const TW* p, int64_t i);
template <> __device__ __forceinline__ float ldw<float>(const float* p, int64_t i) { return p[i]; }
template <> __device__ __forceinline__ float ldw<uint16_t>(const uint16_t* p, int64_t i) { return bf2f(p[i]); }

__device__ __forceinline__ void ldw16(const float* p, float (&o)[16]) {
#pragma unroll
    for (int i = 0; i < 16; i++) o[i] = p[i];
}
__device__ __forceinline__ void ldw16(const uint16_t* p, float (&o)[16]) {
    if (((uintptr_t)p & 15) == 0) {
        const uint4 a = *reinterpret_cast<const uint4*>(p), b = *reinterpret_cast<const uint4*>(p + 8);
        const uint32_t u[8] = {a.x, a.y, a.z, a.w, b.x, b.y, b.z, b.w};
#pragma unroll
        for (int i = 0; i < 8; i++) {
            o[2 * i] = bf2f(u[i] & 0xffffu);
            o[2 * i + 1] = bf2f(u[i] >> 16);
        }
    } else {
#pragma unroll
        for (int i = 0; i < 16; i++) o[i] = bf2f(p[i]);
    }
}

template <typename TW>
__global__ __launch_bounds__(256) void low_rank_log_sigmoid_kernel(const float* in, int64_t ld_in, int rank, const TW* w, const float* bias,
                                                                   float inv_tau, int n, int T, float* out) {
    extern __shared__ float a1[];   // [LR][rank]
    const int t0 = blockIdx.y * LR, nt = min(LR, T - t0), c = blockIdx.x * 256 + threadIdx.x;
    for (int i = threadIdx.x; i < LR * rank; i += 256) {
        const int r = i / rank;
        a1[i] = r < nt ? in[(int64_t)(t0 + r) * ld_in + i % rank] : 0.f;
    }
    __syncthreads();
    if (c >= n) return;
    float z[LR] = {};
    const TW* wr = w + (int64_t)c * rank;
    int k = 0;
    for (; k + 16 <= rank; k += 16) {   // the weights of 16 ranks first, as many independent loads
        float wk[16];
        ldw16(wr + k, wk);
#pragma unroll
        for (int j = 0; j < 16; j++)
#pragma unroll
            for (int r = 0; r < LR; r++) z[r] = fmaf(wk[j], a1[r * rank + k + j], z[r]);
    }
    for (; k < rank; k++) {
        const float wk = ldw<TW>(wr, k);
#pragma unroll
        for (int r = 0; r < LR; r++) z[r] = fmaf(wk, a1[r * rank + k], z[r]);
    }
    const float b = bias[c];
#pragma unroll
    for (int r = 0; r < LR; r++)
        if (r < nt) out[(int64_t)(t0 + r) * n + c] = -softplus(-(z[r] + b)) * inv_tau;
}
int low_rank_log_sigmoid(const float* in, int64_t ld_in, int rank, const void* w, bool w_f32, const float* bias, float tau, int n, int T,
                         float* out, hipStream_t st) {
    QIE_REQUIRE(in && w && bias && out && rank > 0 && n > 0 && tau > 0.f, "low-rank decay: bad arguments");
    const size_t shm = (size_t)LR * rank * 4;
    QIE_REQUIRE(shm <= 60 * 1024, "low-rank decay: rank %d above the kernel's staging", rank);
    dim3 grid((unsigned)((n + 255) / 256), (unsigned)((T + LR - 1) / LR));
    if (w_f32)
        hipLaunchKernelGGL(low_rank_log_sigmoid_kernel<float>, grid, dim3(256), shm, st, in, ld_in, rank, (const float*)w, bias, 1.0f / tau,
                           n, T, out);
    else
        hipLaunchKernelGGL(low_rank_log_sigmoid_kernel<uint16_t>, grid, dim3(256), shm, st, in, ld_in, rank, (const uint16_t*)w, bias,
                           1.0f / tau, n, T, out);
    QIE_LAUNCH_CHECK();
    return 0;
}

}  // namespace lay
}  // namespace qie
