// kr_serve_linear.hip -- linear-recurrence mixers of the batched serving step around their scans (gfx950, wave64): the token shift and the decays of the wkv mixer,
// the preparation of the gated delta rule (convolution, unit vectors, gates), lightning attention's output norm, and the block forms of
// both recurrences for prompt portions.
// Everything is f32 but the storage-type inputs and outputs of the projections.
#include <hip/hip_runtime.h>
#include <math.h>
#include <stdint.h>

#include "kr_device.h"
#include "kr_serve_ops.h"

namespace {
typedef float ln_f4 __attribute__((ext_vector_type(4)));
__device__ __forceinline__ float ln_ld(const float* p) { return *p; }
__device__ __forceinline__ float ln_ld(const uint16_t* p) { return kr_bf16_to_f32(*p); }
__device__ __forceinline__ void ln_st(float* p, float v) { *p = v; }
__device__ __forceinline__ void ln_st(uint16_t* p, float v) { *p = kr_f32_to_bf16(v); }
__device__ __forceinline__ float ln_wave_sum(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o);
    return v;
}

// ---- wkv: the n shifted inputs of a token (KrSvShift): a thread per VC channels of TT consecutive tokens
template <typename T, int VC, int TT>
__global__ void __launch_bounds__(256) ln_shift_kernel(const KrSvShift a, T* __restrict__ out) {
    const int t0 = blockIdx.x * TT, c = (blockIdx.y * 256 + threadIdx.x) * VC;
    if (blockIdx.y == 0) {                                  // the grouped problem's tables
        for (int i = threadIdx.x; i < a.n * TT; i += 256) {
            const int t = t0 + i / a.n, k = i % a.n;
            if (t >= a.T) break;
            a.group[k * a.T + t] = k;
            a.c_rows[k * a.T + t] = k < a.n - 1 ? t * (a.n - 1) + k : (a.n - 1) * a.T + t * a.last_rows;
        }
        if (t0 == 0 && (int)threadIdx.x <= a.n) a.seg[threadIdx.x] = threadIdx.x * a.T;
    }
    if (c >= a.width) return;
    float h[TT + 1][VC];                                    // h[0]: the token before t0
    auto load = [&](const float* p, float* v) {
        if constexpr (VC == 4) { const float4 x = *reinterpret_cast<const float4*>(p); v[0] = x.x; v[1] = x.y; v[2] = x.z; v[3] = x.w; }
        else v[0] = *p;
    };
#pragma unroll
    for (int i = 0; i <= TT; i++) load(a.h32 + (size_t)min(max(t0 + i - 1, 0), a.T - 1) * a.width + c, h[i]);
    float prev[TT][VC];
#pragma unroll
    for (int i = 0; i < TT; i++) {
        const int t = min(t0 + i, a.T - 1), sl = a.slot[t];
        const bool own = t > 0 && a.slot[t - 1] == sl, first = a.pos[t] == 0;      // the token before: a row of this step, nothing, or the request's state
#pragma unroll
        for (int k = 0; k < VC; k++) prev[i][k] = first ? 0.0f : h[i][k];
        if (!own && !first) load(a.state + (size_t)sl * a.width + c, prev[i]);
    }
    for (int n = 0; n < a.n; n++) {
        float mu[VC];
        load(a.mu + (size_t)n * a.width + c, mu);
#pragma unroll
        for (int i = 0; i < TT; i++) {
            if (t0 + i >= a.T) break;
            T* o = out + ((size_t)n * a.T + t0 + i) * a.width + c;
            float v[VC];
#pragma unroll
            for (int k = 0; k < VC; k++) v[k] = __builtin_fmaf(prev[i][k] - h[i + 1][k], mu[k], h[i + 1][k]);
            if constexpr (VC == 4 && sizeof(T) == 2) {
                *reinterpret_cast<uint2*>(o) = make_uint2((uint32_t)kr_f32_to_bf16(v[0]) | ((uint32_t)kr_f32_to_bf16(v[1]) << 16), (uint32_t)kr_f32_to_bf16(v[2]) | ((uint32_t)kr_f32_to_bf16(v[3]) << 16));
            } else if constexpr (VC == 4) *reinterpret_cast<float4*>(o) = make_float4(v[0], v[1], v[2], v[3]);
            else ln_st(o, v[0]);
        }
    }
}

// log decays of TT tokens x 256 channels: tanh of the low-rank rows in LDS, a channel's weights through registers, sixteen ranks at a time
template <typename T, int TT>
__global__ void __launch_bounds__(256) ln_wkv_decay_kernel(const float* __restrict__ z, int ld, const T* __restrict__ w2, const float* __restrict__ w0, int T_, int rank, int cols,
                                                           float* __restrict__ out) {
    constexpr int RB = 64;
    __shared__ __attribute__((aligned(16))) float zs[TT][RB];
    const int t0 = blockIdx.x * TT, c = blockIdx.y * 256 + threadIdx.x, cc = min(c, cols - 1);
    const bool vec = rank % 16 == 0 && ((uintptr_t)w2 & 15) == 0;
    float acc[TT];
#pragma unroll
    for (int i = 0; i < TT; i++) acc[i] = 0.0f;
    for (int r0 = 0; r0 < rank; r0 += RB) {
        const int nr = min(RB, rank - r0);
        __syncthreads();
        for (int i = threadIdx.x; i < TT * RB; i += 256) {
            const int tt = i / RB, r = i - tt * RB;
            zs[tt][r] = (t0 + tt < T_ && r < nr) ? tanhf(z[(size_t)(t0 + tt) * ld + r0 + r]) : 0.0f;
        }
        __syncthreads();
        const T* wr = w2 + (size_t)cc * rank + r0;
        for (int r = 0; r < nr; r += 16) {
            float w[16];
            if (vec) {
                constexpr int VEC = 16 / sizeof(T);
#pragma unroll
                for (int u = 0; u < 16 / VEC; u++) {
                    const uint4 v = *reinterpret_cast<const uint4*>(wr + r + u * VEC);
                    const uint32_t x[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
                    for (int e = 0; e < 4; e++) {
                        if constexpr (sizeof(T) == 2) { w[u * 8 + 2 * e] = __uint_as_float(x[e] << 16); w[u * 8 + 2 * e + 1] = __uint_as_float(x[e] & 0xFFFF0000u); }
                        else w[u * 4 + e] = __uint_as_float(x[e]);
                    }
                }
            } else {
#pragma unroll
                for (int u = 0; u < 16; u++) w[u] = r + u < nr ? ln_ld(wr + r + u) : 0.0f;
            }
#pragma unroll
            for (int tt = 0; tt < TT; tt++)
#pragma unroll
                for (int u = 0; u < 16; u += 4) {
                    const float4 z4 = *reinterpret_cast<const float4*>(&zs[tt][r + u]);
                    acc[tt] = __builtin_fmaf(w[u], z4.x, acc[tt]); acc[tt] = __builtin_fmaf(w[u + 1], z4.y, acc[tt]);
                    acc[tt] = __builtin_fmaf(w[u + 2], z4.z, acc[tt]); acc[tt] = __builtin_fmaf(w[u + 3], z4.w, acc[tt]);
                }
        }
    }
    if (c >= cols) return;
    const float b = w0[c];
#pragma unroll
    for (int tt = 0; tt < TT; tt++) if (t0 + tt < T_) out[(size_t)(t0 + tt) * cols + c] = -expf(acc[tt] + b);
}

// ---- gated delta rule: one wave per (TT consecutive tokens, q / k / v head); channel = lane + 64 i of the head.  NT > 0: that many taps, whose rows pass through
// registers (a row is read once for all the tokens it reaches); NT = 0: any number, read again for every token.
template <int NT, int TT>
__global__ void __launch_bounds__(64) ln_delta_prep_kernel(const KrSvDelta a) {
    const int t0 = blockIdx.x * TT, y = blockIdx.y, lane = threadIdx.x, G = a.kv_heads;
    const bool isv = y >= 2 * G;
    const int n = isv ? a.vdim : a.dim, c0 = isv ? 2 * G * a.dim + (y - 2 * G) * a.vdim : y * a.dim, C = 2 * G * a.dim + a.heads * a.vdim;
    const int taps = NT ? NT : a.taps;
    float ss[TT];
#pragma unroll
    for (int i = 0; i < TT; i++) ss[i] = 0.0f;
    float* o = a.out + (size_t)t0 * C + c0;
    for (int d = lane; d < n; d += 64) {
        const int c = c0 + d;
        const float* w = a.conv + (size_t)c * taps;
        const float* zc = a.z + c;
        if constexpr (NT > 0) {
            float wt[NT], u[TT + NT - 1];                       // u[i]: row t0 - (NT - 1) + i of the step
#pragma unroll
            for (int b = 0; b < NT; b++) wt[b] = w[b];
#pragma unroll
            for (int i = 0; i < TT + NT - 1; i++) u[i] = zc[(size_t)min(max(t0 + i - (NT - 1), 0), a.T - 1) * a.ld];
#pragma unroll
            for (int i = 0; i < TT; i++) {
                const int t = t0 + i, tc = min(t, a.T - 1), p = a.pos[tc], sl = a.slot[tc];
                float r[NT];                                    // r[b]: b positions back
#pragma unroll
                for (int b = 0; b < NT; b++) {
                    r[b] = u[i + NT - 1 - b];
                    if (b > 0) {
                        const bool own = tc - b >= 0 && a.slot[max(tc - b, 0)] == sl;
                        if (p - b < 0) r[b] = 0.0f;
                        else if (!own) r[b] = a.ring[((size_t)sl * NT + (p - b) % NT) * C + c];
                    }
                }
                float acc = wt[NT - 1] * r[0];
#pragma unroll
                for (int b = 1; b < NT; b++) acc = __builtin_fmaf(wt[NT - 1 - b], r[b], acc);
                if (t >= a.T) break;
                if (a.single && NT > 1) a.ring[((size_t)sl * NT + p % NT) * C + c] = r[0];
                const float v = acc / (1.0f + expf(-acc));
                ss[i] = __builtin_fmaf(v, v, ss[i]);
                o[(size_t)i * C + d] = v;
            }
        } else {
#pragma unroll
            for (int i = 0; i < TT; i++) {
                const int t = t0 + i;
                if (t >= a.T) break;
                const int p = a.pos[t], sl = a.slot[t];
                const float u0 = zc[(size_t)t * a.ld];
                float acc = w[taps - 1] * u0;
                for (int b = 1; b < taps && p - b >= 0; b++) {
                    const float u = (t - b >= 0 && a.slot[t - b] == sl) ? zc[(size_t)(t - b) * a.ld] : a.ring[((size_t)sl * taps + (p - b) % taps) * C + c];
                    acc = __builtin_fmaf(w[taps - 1 - b], u, acc);
                }
                if (a.single) a.ring[((size_t)sl * taps + p % taps) * C + c] = u0;
                const float v = acc / (1.0f + expf(-acc));
                ss[i] = __builtin_fmaf(v, v, ss[i]);
                o[(size_t)i * C + d] = v;
            }
        }
    }
    if (!isv) {
        const float qs = y < G ? 1.0f / sqrtf((float)a.dim) : 1.0f;
#pragma unroll
        for (int i = 0; i < TT; i++) {
            if (t0 + i >= a.T) break;
            const float sc = qs / sqrtf(ln_wave_sum(ss[i]) + 1e-6f);
            for (int d = lane; d < n; d += 64) o[(size_t)i * C + d] *= sc;      // a lane's own words
        }
    } else if (lane < TT && t0 + lane < a.T) {
        const int h = y - 2 * G, t = t0 + lane;
        const float zb = a.bz[(size_t)t * a.ld + h], za = a.az[(size_t)t * a.ld + h] + a.dt_bias[h];
        const float sp = fmaxf(za, 0.0f) + log1pf(expf(-fabsf(za)));      // softplus
        a.tok[(size_t)t * a.heads + h] = make_float4(-expf(a.a_log[h]) * sp, 0.0f, 0.0f, 1.0f / (1.0f + expf(-zb)));
    }
}
// the last taps - 1 projected rows of every portion -> the request's ring
__global__ void __launch_bounds__(256) ln_delta_save_kernel(const KrSvDelta a) {
    const int e = blockIdx.x, i = blockIdx.y, c = blockIdx.z * 256 + threadIdx.x, C = 2 * a.kv_heads * a.dim + a.heads * a.vdim;
    const int t = a.ent_off[e + 1] - 1 - i;
    if (c >= C || t < a.ent_off[e]) return;
    a.ring[((size_t)a.slot[t] * a.taps + a.pos[t] % a.taps) * C + c] = a.z[(size_t)t * a.ld + c];
}

// ---- lightning attention: the heads side by side as one row
// NT threads: 256 for prompt-sized steps, 1024 where a row's workgroup is alone on its compute unit
template <typename T, int NT>
__global__ void __launch_bounds__(NT) ln_row_out_kernel(const float* __restrict__ o, int n, const float* __restrict__ w, const float* __restrict__ gate, int gate_ld, float eps, float scale,
                                                        T* __restrict__ out, int out_ld) {
    __shared__ float red[NT / 64];
    const size_t t = blockIdx.x;
    const float* r = o + t * n;
    float ss = 0.0f;
#pragma unroll 4
    for (int c = threadIdx.x; c < n; c += NT) ss = __builtin_fmaf(r[c], r[c], ss);
    ss = ln_wave_sum(ss);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    float all = 0.0f;
#pragma unroll
    for (int i = 0; i < NT / 64; i++) all += red[i];
    const float inv = scale / sqrtf(all / (float)n + eps);
#pragma unroll 4
    for (int c = threadIdx.x; c < n; c += NT) ln_st(out + t * out_ld + c, r[c] * inv * w[c] / (1.0f + expf(-gate[t * gate_ld + c])));
}

// ---- block form of the recurrences with a decay per key channel (gla, wkv), prompt portions: blocks of 64 tokens, four sub-blocks of 16.
// With f_s the sum of the log decays from the start of s's sub-block to s, and tot_m that of a whole sub-block, every weight between two tokens splits into
// exp(e_t) * prod(sub-blocks between) * exp(tot - f_s) (e_t = f_t, or the sum before t where the read-out comes before the write): all three factors are <= 1, so
// strong decays cannot overflow.  Inside a sub-block the split would be exp(e_t - tot) * exp(tot - f_s), whose first factor is >= 1: it is taken while the
// sub-block's sums stay above -60, and below that the sixteen tokens' weights are formed pair by pair.
// gla: log decays from their logits, in place: log sigmoid(z + b) / tau
__global__ void __launch_bounds__(256) ln_gla_log_kernel(float* __restrict__ gz, const float* __restrict__ bias, size_t n, int cols, float inv_tau) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    const float z = gz[i] + bias[i % cols];
    gz[i] = (fminf(z, 0.0f) - log1pf(expf(-fabsf(z)))) * inv_tau;
}
// (1) in parallel over (block, head): f in place of the log decays, the block's own contribution U = sum_s exp(F_last - F_s) k_s v_s^T to a.sbuf, exp(F_last) to a.nbuf
__device__ __forceinline__ int ln_entry_of(const KrSvLin& a, int gc) { int e = 0; while (e + 1 < a.n_entries && a.ent_chunk0[e + 1] <= gc) e++; return e; }
template <int DT>          // 16-row tiles of a head's keys: 4 (dim <= 64) or 8 (dim <= 128)
__global__ void __launch_bounds__(256) ln_chan_local_kernel(const KrSvLin a) {
    constexpr int DP = DT * 16, LK = DP + 16, NG = 256 / DP;      // LDS rows 16 banks apart: the four token rows of a fragment read fall into distinct banks
    extern __shared__ __attribute__((aligned(16))) float lds[];
    float* kt = lds; float* tots = kt + 64 * LK;                  // [64][LK], [4][DP]
    const int gc = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, kq = lane >> 4;
    const int H = a.heads, dim = a.dim, vdim = a.vdim, nct = (vdim + 15) / 16;
    const int e = ln_entry_of(a, gc), tb = a.ent_off[e] + 64 * (gc - a.ent_chunk0[e]), nt = min(64, a.ent_off[e + 1] - tb);
    const int d = tid % DP, grp = tid / DP; const bool dv = d < dim; const int dc = dv ? d : 0;
    float* gz = const_cast<float*>(a.gz) + (size_t)tb * a.gz_ld + (size_t)h * dim + dc;
    const float* kp = a.ksrc + (size_t)tb * a.src_ld + (size_t)h * dim + dc;
    for (int m = grp; m < 4; m += NG) {
        float f[16], k[16];
#pragma unroll
        for (int i = 0; i < 16; i++) { const int s = min(16 * m + i, nt - 1); f[i] = gz[(size_t)s * a.gz_ld]; k[i] = kp[(size_t)s * a.src_ld]; }
        float run = 0.0f;
#pragma unroll
        for (int i = 0; i < 16; i++) {
            const bool ok = dv && 16 * m + i < nt;
            run += ok ? f[i] : 0.0f; f[i] = run;
            if (!ok) k[i] = 0.0f; else gz[(size_t)(16 * m + i) * a.gz_ld] = run;
        }
        tots[m * DP + d] = run;
#pragma unroll
        for (int i = 0; i < 16; i++) kt[(16 * m + i) * LK + d] = k[i] * expf(run - f[i]);
    }
    __syncthreads();
    for (int m = grp; m < 4; m += NG) {
        float after = 0.0f;
        for (int n = m + 1; n < 4; n++) after += tots[n * DP + d];
        const float w = expf(after);
        if (m < 3) {
#pragma unroll
            for (int i = 0; i < 16; i++) kt[(16 * m + i) * LK + d] *= w;
        }
        if (m == 0 && dv) a.nbuf[((size_t)gc * H + h) * dim + d] = expf(after + tots[d]);
    }
    __syncthreads();
    const float* vp = a.vsrc + (size_t)tb * a.src_ld + (size_t)h * vdim;
    float* U = a.sbuf + ((size_t)gc * H + h) * dim * vdim;
    for (int ct = wave; ct < nct; ct += 4) {
        const int c = ct * 16 + r; const bool cv = c < vdim;
        float vv[16];
#pragma unroll
        for (int j = 0; j < 16; j++) { const int s = 4 * j + kq; const float x = vp[(size_t)min(s, nt - 1) * a.src_ld + (cv ? c : 0)]; vv[j] = (cv && s < nt) ? x : 0.0f; }
#pragma unroll
        for (int t = 0; t < DT; t++) {
            if (t * 16 >= dim) break;
            ln_f4 acc = ln_f4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int j = 0; j < 16; j++) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(kt[(4 * j + kq) * LK + t * 16 + r], vv[j], acc, 0, 0, 0);
#pragma unroll
            for (int i = 0; i < 4; i++) { const int dd = t * 16 + 4 * kq + i; if (cv && dd < dim) U[(size_t)dd * vdim + c] = acc[i]; }
        }
    }
}
// (2) element by element over an entry's blocks: the state at the block's start where its contribution stood, S <- exp(F_last) S + U
__global__ void __launch_bounds__(256) ln_chan_scan_kernel(const KrSvLin a) {
    const int e = blockIdx.x, h = blockIdx.y, H = a.heads, dim = a.dim, vdim = a.vdim, idx = blockIdx.z * 256 + threadIdx.x, nS = dim * vdim;
    if (idx >= nS) return;
    const int t0 = a.ent_off[e], nch = (a.ent_off[e + 1] - t0 + 63) / 64, c0 = a.ent_chunk0[e], d = idx / vdim, col = idx - d * vdim;
    float* Sg = a.state + (size_t)a.ent_slot[e] * a.state_stride + ((size_t)h * vdim + col) * dim + d;
    float S = a.pos[t0] == 0 ? 0.0f : *Sg;
    float* p = a.sbuf + ((size_t)c0 * H + h) * nS + idx; const size_t step = (size_t)H * nS;
    const float* g = a.nbuf + ((size_t)c0 * H + h) * dim + d; const size_t gs = (size_t)H * dim;
    for (int c = 0; c < nch; c += 8) {
        float u[8], w[8];
#pragma unroll
        for (int k = 0; k < 8; k++) { const int cc = min(c + k, nch - 1); u[k] = p[(size_t)cc * step]; w[k] = g[(size_t)cc * gs]; }
#pragma unroll
        for (int k = 0; k < 8; k++) if (c + k < nch) { p[(size_t)(c + k) * step] = S; S = __builtin_fmaf(w[k], S, u[k]); }
    }
    *Sg = S;
}
// (3) in parallel over (block, head), wave w = sub-block w: both products transposed (S^T[s][t] = K Q^T, O^T[c][t] = V^T P^T) so that the weights meet the values where the
// first product left them.  The wave's queries stay in registers and collect the decays of the sub-blocks they pass on the way back.
template <int DT, int DB, bool WKV>
__global__ void __launch_bounds__(256) ln_chan_out_kernel(const KrSvLin a) {
    constexpr int DP = DT * 16, LK = DP + 4, LS = DB * 16 + 16;
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int gc = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, kq = lane >> 4;
    const int H = a.heads, dim = a.dim, vdim = a.vdim;
    float* tot = lds; float* et = tot + 4 * DP; float* kd = et + 4 * DP; float* sl = kd;      // [4][DP] twice, [64][LK], later [32][LS] rows of the block's start state
    const int e = ln_entry_of(a, gc), tb = a.ent_off[e] + 64 * (gc - a.ent_chunk0[e]), nt = min(64, a.ent_off[e + 1] - tb);
    const bool active = wave * 16 < nt;
    const int trow = wave * 16 + r; const bool tv = trow < nt;
    const int tc = min(trow, nt - 1);
    // reduction step i of lane group kq takes channel 16 (i / 4) + 4 kq + i % 4: four steps of a lane are 16 contiguous bytes
    const bool vec = dim == DP && ((a.src_ld | a.gz_ld) & 3) == 0 && (((uintptr_t)a.qsrc | (uintptr_t)a.ksrc | (uintptr_t)a.gz | (uintptr_t)a.bonus) & 15) == 0;
    auto ld4 = [&](const float* p, int d) {
        if (vec) return *reinterpret_cast<const float4*>(p + d);
        return make_float4(p[min(d, dim - 1)], p[min(d + 1, dim - 1)], p[min(d + 2, dim - 1)], p[min(d + 3, dim - 1)]);
    };
    const float* fz = a.gz + (size_t)tb * a.gz_ld + (size_t)h * dim;
    const float* kz = a.ksrc + (size_t)tb * a.src_ld + (size_t)h * dim; const float* qz = a.qsrc + (size_t)tb * a.src_ld + (size_t)h * dim;
    const float* vz = a.vsrc + (size_t)tb * a.src_ld + (size_t)h * vdim;
    for (int i = tid; i < 4 * DP; i += 256) {
        const int m = i / DP, d = i - m * DP;
        const float v = (d < dim && 16 * m < nt) ? fz[(size_t)min(16 * m + 15, nt - 1) * a.gz_ld + d] : 0.0f;
        tot[i] = v; et[i] = expf(v);
    }
    float4 q4[DT];
    float bonus = 0.0f;
    {
        const float* qp = qz + (size_t)tc * a.src_ld; const float* kp = kz + (size_t)tc * a.src_ld; const float* fp = fz + (size_t)(WKV ? max(tc - 1, 0) : tc) * a.gz_ld;
        const bool past = !WKV || r > 0;                          // a sub-block's first token reads what the sub-block before left
#pragma unroll
        for (int i = 0; i < DT; i++) {
            const int d = 16 * i + 4 * kq;
            float4 x = ld4(qp, d); const float4 f = ld4(fp, d);
            x.x *= a.q_scale; x.y *= a.q_scale; x.z *= a.q_scale; x.w *= a.q_scale;
            if (d >= dim) x.x = 0.0f; if (d + 1 >= dim) x.y = 0.0f; if (d + 2 >= dim) x.z = 0.0f; if (d + 3 >= dim) x.w = 0.0f;
            if constexpr (WKV) {
                const float4 u = ld4(a.bonus + (size_t)h * dim, d), k = ld4(kp, d);
                bonus = __builtin_fmaf(x.x * u.x, k.x, bonus); bonus = __builtin_fmaf(x.y * u.y, k.y, bonus); bonus = __builtin_fmaf(x.z * u.z, k.z, bonus); bonus = __builtin_fmaf(x.w * u.w, k.w, bonus);
            }
            if (past) { x.x *= expf(f.x); x.y *= expf(f.y); x.z *= expf(f.z); x.w *= expf(f.w); }
            q4[i] = x;
        }
    }
    if constexpr (WKV) { bonus += __shfl_xor(bonus, 16); bonus += __shfl_xor(bonus, 32); }
    __syncthreads();
#pragma unroll 4
    for (int i = tid; i < 64 * (DP / 4); i += 256) {
        const int s = i / (DP / 4), d = 4 * (i - s * (DP / 4)), sc = min(s, nt - 1);
        float4 k = ld4(kz + (size_t)sc * a.src_ld, d); const float4 f = ld4(fz + (size_t)sc * a.gz_ld, d), t4 = *reinterpret_cast<const float4*>(tot + (s >> 4) * DP + d);
        const bool ok = s < nt;
        k.x = ok && d < dim ? k.x * expf(t4.x - f.x) : 0.0f; k.y = ok && d + 1 < dim ? k.y * expf(t4.y - f.y) : 0.0f;
        k.z = ok && d + 2 < dim ? k.z * expf(t4.z - f.z) : 0.0f; k.w = ok && d + 3 < dim ? k.w * expf(t4.w - f.w) : 0.0f;
        *reinterpret_cast<float4*>(kd + s * LK + d) = k;
    }
    float big = 0.0f;
#pragma unroll
    for (int i = 0; i < DT; i++) { const float4 t4 = *reinterpret_cast<const float4*>(tot + wave * DP + 16 * i + 4 * kq); big = fmaxf(big, fmaxf(fmaxf(-t4.x, -t4.y), fmaxf(-t4.z, -t4.w))); }
    big = fmaxf(big, __shfl_xor(big, 16)); big = fmaxf(big, __shfl_xor(big, 32));      // the same in every lane of a wave: lanes of one group share their channels
    __syncthreads();
    ln_f4 acc[DB];
#pragma unroll
    for (int c = 0; c < DB; c++) acc[c] = ln_f4{0.0f, 0.0f, 0.0f, 0.0f};
    if (active) {
#pragma nounroll
        for (int j = wave; j >= 0; j--) {
            size_t srow[4]; float vf[4][DB];                      // the value rows of the tile's keys: requested before the first product
#pragma unroll
            for (int i = 0; i < 4; i++) srow[i] = (size_t)min(16 * j + 4 * kq + i, nt - 1) * a.src_ld;
#pragma unroll
            for (int i = 0; i < 4; i++)
#pragma unroll
                for (int c = 0; c < DB; c++) vf[i][c] = vz[srow[i] + min(c * 16 + r, vdim - 1)];
            ln_f4 st = ln_f4{0.0f, 0.0f, 0.0f, 0.0f};
            const float* krow = kd + (16 * j + r) * LK + 4 * kq;
            const float* ep = et + j * DP + 4 * kq;
            if (j == wave && big > 60.0f) {
                for (int d = 0; d < dim; d++) {
                    const float x = qz[(size_t)tc * a.src_ld + d] * a.q_scale;
                    const float ev = WKV ? (r > 0 ? fz[(size_t)max(tc - 1, 0) * a.gz_ld + d] : 0.0f) : fz[(size_t)tc * a.gz_ld + d];
#pragma unroll
                    for (int i = 0; i < 4; i++) {
                        const int s = min(16 * j + 4 * kq + i, nt - 1);
                        st[i] = __builtin_fmaf(x * kz[(size_t)s * a.src_ld + d], expf(fminf(ev - fz[(size_t)s * a.gz_ld + d], 0.0f)), st[i]);      // pairs the mask below drops may have a positive difference
                    }
                }
            } else {
                // inside the own sub-block the queries go back to its end first (exp(e_t - tot)); on the way to the one before an earlier one they take that one's decay along
                const bool own = j == wave;
#pragma unroll
                for (int i = 0; i < DT; i++) {
                    const float4 k4 = *reinterpret_cast<const float4*>(krow + 16 * i), e4 = *reinterpret_cast<const float4*>(ep + 16 * i);
                    const float4 x = own ? make_float4(q4[i].x / e4.x, q4[i].y / e4.y, q4[i].z / e4.z, q4[i].w / e4.w) : q4[i];
                    st = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.x, x.x, st, 0, 0, 0); st = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.y, x.y, st, 0, 0, 0);
                    st = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.z, x.z, st, 0, 0, 0); st = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.w, x.w, st, 0, 0, 0);
                    if (!own) q4[i] = make_float4(q4[i].x * e4.x, q4[i].y * e4.y, q4[i].z * e4.z, q4[i].w * e4.w);
                }
            }
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int s = 16 * j + 4 * kq + i;
                if (j == wave) { if (WKV && s == trow) st[i] = bonus; else if (s > trow) st[i] = 0.0f; }
                if (!tv) st[i] = 0.0f;
            }
#pragma unroll
            for (int i = 0; i < 4; i++)
#pragma unroll
                for (int c = 0; c < DB; c++) acc[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(vf[i][c], st[i], acc[c], 0, 0, 0);
        }
    }
    const float* Sc = a.sbuf + ((size_t)gc * H + h) * dim * vdim;
#pragma unroll
    for (int p0 = 0; p0 < DP; p0 += 32) {           // the state's share: passes over 32 of its rows
        if (p0 >= dim) break;
        const int rows = min(32, dim - p0);
        __syncthreads();
        if ((vdim & 3) == 0) {
            const int v4 = vdim >> 2;
            for (int i = tid; i < rows * v4; i += 256) { const int rr = i / v4, c4 = i - rr * v4; *reinterpret_cast<float4*>(sl + rr * LS + 4 * c4) = *reinterpret_cast<const float4*>(Sc + (size_t)(p0 + rr) * vdim + 4 * c4); }
        } else {
            for (int i = tid; i < rows * vdim; i += 256) { const int rr = i / vdim, cc = i - rr * vdim; sl[rr * LS + cc] = Sc[(size_t)(p0 + rr) * vdim + cc]; }
        }
        __syncthreads();
        if (active) {
#pragma unroll
            for (int i = 0; i < 8; i++) {
                const int lr = 16 * (i >> 2) + 4 * kq + (i & 3);
                const float4 qq = q4[p0 / 16 + (i >> 2)];
                const float qi = (i & 3) == 0 ? qq.x : (i & 3) == 1 ? qq.y : (i & 3) == 2 ? qq.z : qq.w;      // zero past dim
                const float* srow = sl + min(lr, rows - 1) * LS + r;
#pragma unroll
                for (int c = 0; c < DB; c++) acc[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(srow[c * 16], qi, acc[c], 0, 0, 0);      // columns past vdim are not stored
            }
        }
    }
    if (!active || !tv) return;
    float* o = a.o + (size_t)(tb + trow) * H * vdim + (size_t)h * vdim;
#pragma unroll
    for (int c = 0; c < DB; c++) {
        const int c0 = c * 16 + 4 * kq;
        if ((vdim & 3) == 0) { if (c0 < vdim) *reinterpret_cast<float4*>(o + c0) = make_float4(acc[c][0], acc[c][1], acc[c][2], acc[c][3]); }
        else {
#pragma unroll
            for (int i = 0; i < 4; i++) if (c0 + i < vdim) o[c0 + i] = acc[c][i];
        }
    }
}

// ---- block form of the gated delta rule.  Within a block of 64 tokens, F the running sum of the log decays and S the state at its start:
//   u_t = b_t (v_t - e^{F_t} S^T k_t - sum_(s < t) e^{F_t - F_s} (k_s . k_t) u_s)   <=>   (1 + L) U = diag(b) V - diag(b e^F) K S,   L[t][s] = b_t e^{F_t - F_s} k_t . k_s  (s < t)
// so U = X - Y S with X = M diag(b) V and Y = M diag(b e^F) K, M = (1 + L)^-1, which do not know the state.  (1) in parallel over (block, head): L on the matrix instruction;
// M tile by tile -- the four 16 x 16 tiles on the diagonal by substitution (wave w: tile w, a lane per column), those below from M_ij = -M_ii sum_(j <= k < i) L_ik M_kj, the
// inner sum staying in the accumulators, which hold it exactly as the outer product's operand -- then X and Y.  X replaces v, Y goes to a.aux; tok becomes (F, -F, e^F, b).
__global__ void __launch_bounds__(256) ln_delta_solve_kernel(const KrSvLin a) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int gc = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, kq = lane >> 4;
    const int H = a.heads, dim = a.dim, vdim = a.vdim, dimp = ((dim + 15) / 16) * 16, LK = dimp + 4, hq = h / a.qk_group;
    constexpr int LL = 68;
    float* ks = lds; float* Lm = ks + 64 * LK; float* Mm = Lm + 64 * LL; float* Fs = Mm + 64 * LL; float* bs = Fs + 64;      // [64][LK], [64][LL] twice, [64], [64]
    const int e = ln_entry_of(a, gc), tb = a.ent_off[e] + 64 * (gc - a.ent_chunk0[e]), nt = min(64, a.ent_off[e + 1] - tb);
    const float* kz = a.ksrc + (size_t)tb * a.src_ld + (size_t)hq * dim;
    float* vz = const_cast<float*>(a.vsrc) + (size_t)tb * a.src_ld + (size_t)h * vdim;
    for (int i = tid; i < 64 * dimp; i += 256) { const int s = i / dimp, d = i - s * dimp; ks[s * LK + d] = (s < nt && d < dim) ? kz[(size_t)s * a.src_ld + d] : 0.0f; }
    if (wave == 0) {
        const size_t ti = (size_t)(tb + min(lane, nt - 1)) * H + h;
        const float4 tk = a.tok[ti];
        float F = lane < nt ? tk.x : 0.0f;
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) { const float up = __shfl_up(F, o); if (lane >= o) F += up; }
        Fs[lane] = F; bs[lane] = lane < nt ? tk.w : 0.0f;
        if (lane < nt) a.tok[ti] = make_float4(F, -F, expf(F), tk.w);
    }
    __syncthreads();
    auto mm = [](const float4& p, const float4& q, ln_f4 c) {      // four reduction steps: lane group kq holds elements 4 kq .. 4 kq + 3 of both operands
        c = __builtin_amdgcn_mfma_f32_16x16x4f32(p.x, q.x, c, 0, 0, 0); c = __builtin_amdgcn_mfma_f32_16x16x4f32(p.y, q.y, c, 0, 0, 0);
        c = __builtin_amdgcn_mfma_f32_16x16x4f32(p.z, q.z, c, 0, 0, 0); return __builtin_amdgcn_mfma_f32_16x16x4f32(p.w, q.w, c, 0, 0, 0);
    };
    const ln_f4 zero = ln_f4{0.0f, 0.0f, 0.0f, 0.0f};
    for (int ct = 0; ct <= wave; ct++) {            // tile (wave, ct) of K K^T: rows t = 16 wave + 4 kq + i, columns s = 16 ct + r
        ln_f4 acc = zero;
        const float* ka = ks + (16 * wave + r) * LK + 4 * kq; const float* kb = ks + (16 * ct + r) * LK + 4 * kq;
        for (int d = 0; d < dimp; d += 16) acc = mm(*reinterpret_cast<const float4*>(ka + d), *reinterpret_cast<const float4*>(kb + d), acc);
        const int s = 16 * ct + r;
#pragma unroll
        for (int i = 0; i < 4; i++) { const int t = 16 * wave + 4 * kq + i; Lm[t * LL + s] = s < t ? bs[t] * expf(Fs[t] - Fs[s]) * acc[i] : 0.0f; }
    }
    __syncthreads();
    {
        const float* Ld = Lm + 16 * wave * LL + 16 * wave;
        float x[16];
#pragma unroll
        for (int t = 0; t < 16; t++) {
            float v = t == r ? 1.0f : 0.0f;
#pragma unroll
            for (int s = 0; s < t; s++) v = __builtin_fmaf(-Ld[t * LL + s], x[s], v);
            x[t] = v;
        }
        if (kq == 0) {
#pragma unroll
            for (int t = 0; t < 16; t++) Mm[(16 * wave + t) * LL + 16 * wave + r] = x[t];
        }
    }
    __syncthreads();
    for (int dist = 1; dist < 4; dist++) {
        const int j = wave, i = j + dist;
        if (i < 4) {
            ln_f4 acc = zero;
            for (int k = j; k < i; k++) {
                const float* mk = Mm + (16 * k + 4 * kq) * LL + 16 * j + r;
                acc = mm(*reinterpret_cast<const float4*>(Lm + (16 * i + r) * LL + 16 * k + 4 * kq), make_float4(mk[0], mk[LL], mk[2 * LL], mk[3 * LL]), acc);
            }
            ln_f4 m = mm(*reinterpret_cast<const float4*>(Mm + (16 * i + r) * LL + 16 * i + 4 * kq), make_float4(acc[0], acc[1], acc[2], acc[3]), zero);
#pragma unroll
            for (int u = 0; u < 4; u++) Mm[(16 * i + 4 * kq + u) * LL + 16 * j + r] = -m[u];
        }
        __syncthreads();
    }
    // X, then Y: sixteen columns at a time, four row tiles of 16 (i + 1) reduction rows each
    const int nv = (vdim + 15) / 16, nk = dimp / 16;
    for (int ct = wave; ct < nv + nk; ct += 4) {
        const bool isv = ct < nv; const int c = (isv ? ct : ct - nv) * 16 + r; const bool cv = c < (isv ? vdim : dim);
        float b[16];
#pragma unroll
        for (int j = 0; j < 16; j++) {
            const int s = 16 * (j >> 2) + 4 * kq + (j & 3);
            if (isv) { const float x = vz[(size_t)min(s, nt - 1) * a.src_ld + (cv ? c : 0)]; b[j] = (cv && s < nt) ? x * bs[s] : 0.0f; }
            else b[j] = ks[s * LK + c] * bs[s] * expf(Fs[s]);
        }
        float* dst = isv ? vz + c : a.aux + (size_t)tb * H * dim + (size_t)h * dim + c;
        const size_t step = isv ? (size_t)a.src_ld : (size_t)H * dim;
#pragma unroll
        for (int i = 0; i < 4; i++) {
            ln_f4 acc = zero;
#pragma unroll
            for (int k = 0; k <= i; k++) acc = mm(*reinterpret_cast<const float4*>(Mm + (16 * i + r) * LL + 16 * k + 4 * kq), make_float4(b[4 * k], b[4 * k + 1], b[4 * k + 2], b[4 * k + 3]), acc);
#pragma unroll
            for (int u = 0; u < 4; u++) { const int t = 16 * i + 4 * kq + u; if (cv && t < nt) dst[(size_t)t * step] = acc[u]; }
        }
    }
}
// (2) block after block of an entry, one workgroup per (entry, head, 16 value columns): U = X - Y S (wave w: tokens 16 w ..), then S <- e^{F_last} S + sum_s e^{F_last - F_s} k_s u_s^T
// (wave w: NW tiles of key rows, row 16 NW w + NW r + n in tile n, so that a lane's rows stand together in memory).  S lives in the accumulators and, as the next block's
// operand, in LDS; the operands of the next block are requested before the current one is worked on.  Leaves S at the block's start in a.sbuf and U in place of v; the outputs
// are sv_lin_cout_kernel's.
template <int DT, bool VEC>          // 16-row tiles of a head's keys, 4 or 8; VEC: dim fills them and the rows are 16-byte aligned
__global__ void __launch_bounds__(256) ln_delta_state_kernel(const KrSvLin a) {
    constexpr int DP = DT * 16, NW = DT / 4, LS = 20;      // LDS rows of 16 columns, 20 floats apart
    __shared__ __attribute__((aligned(16))) float Sl[DP * LS], Ul[64 * LS];
    const int e = blockIdx.x, h = blockIdx.y, cb = blockIdx.z, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, kq = lane >> 4;
    const int H = a.heads, dim = a.dim, vdim = a.vdim, hq = h / a.qk_group, col = cb * 16 + r; const bool cv = col < vdim; const int colc = cv ? col : 0;
    const int t0 = a.ent_off[e], t1 = a.ent_off[e + 1], nch = (t1 - t0 + 63) / 64, c0 = a.ent_chunk0[e];
    const bool fresh = a.pos[t0] == 0;
    float* Sg = a.state + (size_t)a.ent_slot[e] * a.state_stride + ((size_t)h * vdim + colc) * dim;
    auto drow = [&](int n, int i) { return 16 * NW * wave + NW * (4 * kq + i) + n; };      // the key row of accumulator i of tile n
    ln_f4 S[NW];
#pragma unroll
    for (int n = 0; n < NW; n++)
#pragma unroll
        for (int i = 0; i < 4; i++) { const int d = drow(n, i); const float v = Sg[VEC ? d : min(d, dim - 1)]; S[n][i] = (!fresh && cv && (VEC || d < dim)) ? v : 0.0f; }
    float y[2][DP / 4], kk[2][16][NW], xv[2][4], fs[2][4], fl[2];
    auto fetch = [&](int b, int c) {
        const int tb = t0 + 64 * c, nt = min(64, t1 - tb);
        const float* yp = a.aux + (size_t)(tb + min(16 * wave + r, nt - 1)) * H * dim + (size_t)h * dim;
#pragma unroll
        for (int i = 0; i < DT; i++) {
            const int d = 16 * i + 4 * kq;
            if constexpr (VEC) { const float4 v = *reinterpret_cast<const float4*>(yp + d); y[b][4 * i] = v.x; y[b][4 * i + 1] = v.y; y[b][4 * i + 2] = v.z; y[b][4 * i + 3] = v.w; }
            else {
#pragma unroll
                for (int u = 0; u < 4; u++) y[b][4 * i + u] = yp[min(d + u, dim - 1)];      // meets a zero row of S past dim
            }
        }
        const float* kp = a.ksrc + (size_t)tb * a.src_ld + (size_t)hq * dim;
        const int d0 = 16 * NW * wave + NW * r;
#pragma unroll
        for (int j = 0; j < 16; j++) {
            const float* kr = kp + (size_t)min(4 * j + kq, nt - 1) * a.src_ld;
            if constexpr (VEC && NW == 2) { const float2 v = *reinterpret_cast<const float2*>(kr + d0); kk[b][j][0] = v.x; kk[b][j][NW - 1] = v.y; }
            else {
#pragma unroll
                for (int n = 0; n < NW; n++) kk[b][j][n] = kr[VEC ? d0 + n : min(d0 + n, dim - 1)];
            }
        }
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int s = min(16 * wave + 4 * kq + i, nt - 1);
            xv[b][i] = a.vsrc[(size_t)(tb + s) * a.src_ld + (size_t)h * vdim + colc]; fs[b][i] = a.tok[(size_t)(tb + s) * H + h].x;
        }
        fl[b] = a.tok[(size_t)(tb + nt - 1) * H + h].x;
    };
    auto block = [&](int b, int c) {
        const int tb = t0 + 64 * c, nt = min(64, t1 - tb);
        float* sb = a.sbuf + (((size_t)(c0 + c) * H + h) * dim) * vdim + col;
#pragma unroll
        for (int n = 0; n < NW; n++)
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int d = drow(n, i);
                Sl[d * LS + r] = (VEC || d < dim) ? S[n][i] : 0.0f;
                if (cv && (VEC || d < dim)) sb[(size_t)d * vdim] = S[n][i];
            }
        __syncthreads();
        ln_f4 u = ln_f4{0.0f, 0.0f, 0.0f, 0.0f}, u1 = u;      // two chains: a dependent product waits for the one before
        float sv[2][8];                                      // the state's rows, eight steps read ahead of the eight that are multiplied
        auto read8 = [&](float (&v)[8], int i0) {
#pragma unroll
            for (int k = 0; k < 8; k++) v[k] = Sl[(16 * ((i0 + k) >> 2) + 4 * kq + (k & 3)) * LS + r];
        };
        read8(sv[0], 0);
#pragma unroll
        for (int i = 0; i < DP / 4; i += 8) {
            if (i + 8 < DP / 4) read8(sv[((i >> 3) + 1) & 1], i + 8);
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int k = 0; k < 8; k += 2) {
                u = __builtin_amdgcn_mfma_f32_16x16x4f32(y[b][i + k], sv[(i >> 3) & 1][k], u, 0, 0, 0);
                u1 = __builtin_amdgcn_mfma_f32_16x16x4f32(y[b][i + k + 1], sv[(i >> 3) & 1][k + 1], u1, 0, 0, 0);
            }
        }
        u += u1;
        float* up = const_cast<float*>(a.vsrc) + (size_t)tb * a.src_ld + (size_t)h * vdim + col;
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int s = 16 * wave + 4 * kq + i; const bool ok = s < nt && cv;
            const float v = ok ? xv[b][i] - u[i] : 0.0f;
            Ul[s * LS + r] = v * expf(fl[b] - fs[b][i]);
            if (ok) up[(size_t)s * a.src_ld] = v;
        }
        const float dec = expf(fl[b]);
#pragma unroll
        for (int n = 0; n < NW; n++) S[n] *= dec;
        __syncthreads();
        float uu[16];
#pragma unroll
        for (int j = 0; j < 16; j++) uu[j] = Ul[(4 * j + kq) * LS + r];
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int j = 0; j < 16; j++)
#pragma unroll
            for (int n = 0; n < NW; n++) S[n] = __builtin_amdgcn_mfma_f32_16x16x4f32(kk[b][j][n], uu[j], S[n], 0, 0, 0);
    };
    // blocks in pairs, every request unconditional (past the last block it repeats that one): the wait for a block's operands then leaves the next block's in flight
    int c = 0;
    fetch(0, 0);
    if (nch & 1) { block(0, 0); c = 1; fetch(0, min(1, nch - 1)); }
    for (; c < nch; c += 2) {
        fetch(1, c + 1);
        block(0, c);
        fetch(0, min(c + 2, nch - 1));
        block(1, c + 1);
    }
#pragma unroll
    for (int n = 0; n < NW; n++)
#pragma unroll
        for (int i = 0; i < 4; i++) { const int d = drow(n, i); if (cv && (VEC || d < dim)) Sg[d] = S[n][i]; }
}
}  // namespace

bool kr_sv_lin_blocks_fit(int dim, int vdim) { return dim <= 128 && vdim <= 128; }
void kr_sv_lin_chan_blocks(const KrSvLin& a, hipStream_t st) {
    if (a.T <= 0 || a.n_entries <= 0 || a.n_chunks <= 0) return;
    const dim3 g(a.n_chunks, a.heads);
#define LN_LDS(K_, B_) do { if ((B_) > 48 * 1024) (void)hipFuncSetAttribute((const void*)K_, hipFuncAttributeMaxDynamicSharedMemorySize, (int)(B_)); } while (0)
    if (a.kind == 4) {
        const size_t n = (size_t)a.T * a.heads * a.dim;
        hipLaunchKernelGGL(ln_gla_log_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, st, const_cast<float*>(a.gz), a.gz_bias, n, a.heads * a.dim, a.inv_tau);
    }
    if (a.dim <= 64) { const size_t b = (size_t)(64 * 80 + 4 * 64) * 4; hipLaunchKernelGGL(ln_chan_local_kernel<4>, g, dim3(256), b, st, a); }
    else { const size_t b = (size_t)(64 * 144 + 4 * 128) * 4; LN_LDS(ln_chan_local_kernel<8>, b); hipLaunchKernelGGL(ln_chan_local_kernel<8>, g, dim3(256), b, st, a); }
    hipLaunchKernelGGL(ln_chan_scan_kernel, dim3(a.n_entries, a.heads, (a.dim * a.vdim + 255) / 256), dim3(256), 0, st, a);
#define LN_CO(DT_, DB_, W_) do { const size_t b_ = (size_t)(8 * DT_ * 16 + (64 * (DT_ * 16 + 4) > 32 * (DB_ * 16 + 16) ? 64 * (DT_ * 16 + 4) : 32 * (DB_ * 16 + 16))) * 4; \
        LN_LDS((ln_chan_out_kernel<DT_, DB_, W_>), b_); hipLaunchKernelGGL((ln_chan_out_kernel<DT_, DB_, W_>), g, dim3(256), b_, st, a); } while (0)
#define LN_CO_W(DT_, DB_) do { if (a.kind == 7) LN_CO(DT_, DB_, true); else LN_CO(DT_, DB_, false); } while (0)
    if (a.dim <= 64) { if (a.vdim <= 64) LN_CO_W(4, 4); else LN_CO_W(4, 8); } else { if (a.vdim <= 64) LN_CO_W(8, 4); else LN_CO_W(8, 8); }
#undef LN_CO_W
#undef LN_CO
}
void kr_sv_delta_blocks(const KrSvLin& a, hipStream_t st) {
    if (a.T <= 0 || a.n_entries <= 0 || a.n_chunks <= 0) return;
    const size_t lds = ((size_t)64 * (((a.dim + 15) / 16) * 16 + 4) + 2 * 64 * 68 + 128) * 4;
    LN_LDS(ln_delta_solve_kernel, lds);
    hipLaunchKernelGGL(ln_delta_solve_kernel, dim3(a.n_chunks, a.heads), dim3(256), lds, st, a);
    const dim3 gs(a.n_entries, a.heads, (a.vdim + 15) / 16);
    const bool vec = (a.dim == 64 || a.dim == 128) && (a.src_ld & 3) == 0 && (((uintptr_t)a.ksrc | (uintptr_t)a.aux) & 15) == 0;
    if (a.dim <= 64) { if (vec) hipLaunchKernelGGL((ln_delta_state_kernel<4, true>), gs, dim3(256), 0, st, a); else hipLaunchKernelGGL((ln_delta_state_kernel<4, false>), gs, dim3(256), 0, st, a); }
    else { if (vec) hipLaunchKernelGGL((ln_delta_state_kernel<8, true>), gs, dim3(256), 0, st, a); else hipLaunchKernelGGL((ln_delta_state_kernel<8, false>), gs, dim3(256), 0, st, a); }
    kr_sv_lin_block_out(a, st);
}

void kr_sv_shift(const KrSvShift& a, bool f32, hipStream_t st) {
    if (a.T <= 0) return;
#define LN_SH(T_, VC_, TT_) hipLaunchKernelGGL((ln_shift_kernel<T_, VC_, TT_>), dim3((a.T + TT_ - 1) / TT_, (a.width / VC_ + 255) / 256), dim3(256), 0, st, a, (T_*)a.out)
#define LN_SH_T(T_) do { if (a.width % 4) LN_SH(T_, 1, 1); else if (a.T <= 64) LN_SH(T_, 4, 1); else LN_SH(T_, 4, 4); } while (0)
    if (f32) LN_SH_T(float); else LN_SH_T(uint16_t);
#undef LN_SH_T
#undef LN_SH
}
void kr_sv_wkv_decay(const float* z, int ld, const void* w2, bool f32, const float* w0, int T, int rank, int cols, float* out, hipStream_t st) {
    if (T <= 0) return;
#define LN_DEC(TT_) do { const dim3 grid((T + TT_ - 1) / TT_, (cols + 255) / 256); \
        if (f32) hipLaunchKernelGGL((ln_wkv_decay_kernel<float, TT_>), grid, dim3(256), 0, st, z, ld, (const float*)w2, w0, T, rank, cols, out); \
        else hipLaunchKernelGGL((ln_wkv_decay_kernel<uint16_t, TT_>), grid, dim3(256), 0, st, z, ld, (const uint16_t*)w2, w0, T, rank, cols, out); } while (0)
    if (T <= 64) LN_DEC(1); else LN_DEC(16);
#undef LN_DEC
}
void kr_sv_delta_prep(const KrSvDelta& a, hipStream_t st) {
    if (a.T <= 0) return;
#define LN_DP(NT_, TT_) hipLaunchKernelGGL((ln_delta_prep_kernel<NT_, TT_>), dim3((a.T + TT_ - 1) / TT_, 2 * a.kv_heads + a.heads), dim3(64), 0, st, a)
#define LN_DP_T(NT_) do { if (a.T <= 64) LN_DP(NT_, 1); else LN_DP(NT_, 8); } while (0)
    switch (a.taps) { case 1: LN_DP_T(1); break; case 2: LN_DP_T(2); break; case 3: LN_DP_T(3); break; case 4: LN_DP_T(4); break; default: LN_DP_T(0); break; }
#undef LN_DP_T
#undef LN_DP
    const int C = 2 * a.kv_heads * a.dim + a.heads * a.vdim;
    if (!a.single && a.taps > 1) hipLaunchKernelGGL(ln_delta_save_kernel, dim3(a.n_entries, a.taps - 1, (C + 255) / 256), dim3(256), 0, st, a);
}
void kr_sv_row_out(const float* o, int n, const float* w, const float* gate, int gate_ld, float eps, float scale, void* out, int out_ld, bool f32, int T, hipStream_t st) {
    if (T <= 0) return;
#define LN_RO(T_, NT_) hipLaunchKernelGGL((ln_row_out_kernel<T_, NT_>), dim3(T), dim3(NT_), 0, st, o, n, w, gate, gate_ld, eps, scale, (T_*)out, out_ld)
    if (f32) { if (T <= 64) LN_RO(float, 1024); else LN_RO(float, 256); }
    else { if (T <= 64) LN_RO(uint16_t, 1024); else LN_RO(uint16_t, 256); }
#undef LN_RO
}
