// kr_serve_linear.hip -- linear-recurrence mixers of the batched serving step around their scans (gfx950, wave64): the token shift and the decays of the wkv mixer,
// the preparation of the gated delta rule (convolution, unit vectors, gates), lightning attention's preparation and output norm.
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

// ---- wkv: the n shifted inputs of a token (KrSvShift): one thread per (token, channel)
template <typename T>
__global__ void __launch_bounds__(256) ln_shift_kernel(const KrSvShift a, T* __restrict__ out) {
    const int t = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
    if (blockIdx.y == 0 && (int)threadIdx.x < a.n) {        // the grouped problem's tables
        const int i = threadIdx.x, r = i * a.T + t;
        a.group[r] = i;
        a.c_rows[r] = i < a.n - 1 ? t * (a.n - 1) + i : (a.n - 1) * a.T + t * a.last_rows;
        if (t == 0) { a.seg[i] = i * a.T; if (i == 0) a.seg[a.n] = a.n * a.T; }
    }
    if (c >= a.width) return;
    const int p = a.pos[t], sl = a.slot[t];
    const float h = a.h32[(size_t)t * a.width + c];
    float prev = 0.0f;
    if (p > 0) prev = (t > 0 && a.slot[t - 1] == sl) ? a.h32[(size_t)(t - 1) * a.width + c] : a.state[(size_t)sl * a.width + c];
    const float d = prev - h;
    for (int i = 0; i < a.n; i++) ln_st(out + ((size_t)i * a.T + t) * a.width + c, __builtin_fmaf(d, a.mu[(size_t)i * a.width + c], h));
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

// ---- gated delta rule: one wave per (token, q / k / v head).  The head's channels stay in registers (channel = lane + 64 i)
__global__ void __launch_bounds__(64) ln_delta_prep_kernel(const KrSvDelta a) {
    const int t = blockIdx.x, y = blockIdx.y, lane = threadIdx.x, G = a.kv_heads;
    const bool isv = y >= 2 * G;
    const int n = isv ? a.vdim : a.dim, c0 = isv ? 2 * G * a.dim + (y - 2 * G) * a.vdim : y * a.dim, C = 2 * G * a.dim + a.heads * a.vdim;
    const int p = a.pos[t], sl = a.slot[t], taps = a.taps;
    float v[8], ss = 0.0f;
#pragma unroll
    for (int i = 0; i < 8; i++) {
        const int d = lane + 64 * i;
        v[i] = 0.0f;
        if (d < n) {
            const int c = c0 + d;
            const float* w = a.conv + (size_t)c * taps;
            const float u0 = a.z[(size_t)t * a.ld + c];
            float acc = w[taps - 1] * u0;
            for (int b = 1; b < taps; b++) {      // b positions back
                if (p - b < 0) break;
                const float u = (t - b >= 0 && a.slot[t - b] == sl) ? a.z[(size_t)(t - b) * a.ld + c] : a.ring[((size_t)sl * taps + (p - b) % taps) * C + c];
                acc = __builtin_fmaf(w[taps - 1 - b], u, acc);
            }
            if (a.single && taps > 1) a.ring[((size_t)sl * taps + p % taps) * C + c] = u0;
            v[i] = acc / (1.0f + expf(-acc));
            ss = __builtin_fmaf(v[i], v[i], ss);
        }
    }
    float sc = 1.0f;
    if (!isv) { sc = 1.0f / sqrtf(ln_wave_sum(ss) + 1e-6f); if (y < G) sc *= 1.0f / sqrtf((float)a.dim); }
    float* o = a.out + (size_t)t * C + c0;
#pragma unroll
    for (int i = 0; i < 8; i++) { const int d = lane + 64 * i; if (d < n) o[d] = v[i] * sc; }
    if (isv && lane == 0) {
        const int h = y - 2 * G;
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

// ---- lightning attention
__global__ void __launch_bounds__(256) ln_lt_prep_kernel(float* __restrict__ z, int ld, int cols, const float* __restrict__ decay, int heads, float4* __restrict__ tok) {
    const size_t t = blockIdx.x; const int c = blockIdx.y * 256 + threadIdx.x;
    if (c < heads) tok[t * heads + c] = make_float4(fmaxf(logf(decay[c]), -1.0e4f), 0.0f, 0.0f, 0.0f);
    if (c < cols) { const float v = z[t * ld + c]; z[t * ld + c] = v / (1.0f + expf(-v)); }
}
template <typename T>
__global__ void __launch_bounds__(256) ln_row_out_kernel(const float* __restrict__ o, int n, const float* __restrict__ w, const float* __restrict__ gate, int gate_ld, float eps, float scale,
                                                         T* __restrict__ out, int out_ld) {
    __shared__ float red[4];
    const size_t t = blockIdx.x;
    const float* r = o + t * n;
    float ss = 0.0f;
    for (int c = threadIdx.x; c < n; c += 256) ss = __builtin_fmaf(r[c], r[c], ss);
    ss = ln_wave_sum(ss);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    const float inv = scale / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)n + eps);
    for (int c = threadIdx.x; c < n; c += 256) ln_st(out + t * out_ld + c, r[c] * inv * w[c] / (1.0f + expf(-gate[t * gate_ld + c])));
}
// ---- block form of the recurrences with a decay per key channel (gla, wkv), prompt portions: blocks of 64 tokens, four sub-blocks of 16.
// With f_s the sum of the log decays from the start of s's sub-block to s, and tot_m that of a whole sub-block, every weight between two tokens splits into
// exp(e_t) * prod(sub-blocks between) * exp(tot - f_s) (e_t = f_t, or the sum before t where the read-out comes before the write): all three factors are <= 1, so
// strong decays cannot overflow.  Inside a sub-block the split would be exp(e_t - tot) * exp(tot - f_s), whose first factor is >= 1: it is taken while the
// sub-block's sums stay above -60, and below that the sixteen tokens' weights are formed pair by pair.
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
// first product left them.  The wave's queries live in LDS, one word per (step, lane), and collect the decays of the sub-blocks they pass on the way back.
template <int DB, bool WKV>
__global__ void __launch_bounds__(256) ln_chan_out_kernel(const KrSvLin a) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int gc = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, kq = lane >> 4;
    const int H = a.heads, dim = a.dim, vdim = a.vdim, dimp = ((dim + 15) / 16) * 16, dq = dimp / 4, LK = dimp + 4, LS = ((vdim + 31) / 32) * 32 + 16;
    float* kd = lds; float* tot = kd + 64 * LK; float* et = tot + 4 * dimp; float* sl = et + 4 * dimp; float* qs = sl + 32 * LS + (size_t)wave * dq * 64;
    const int e = ln_entry_of(a, gc), tb = a.ent_off[e] + 64 * (gc - a.ent_chunk0[e]), nt = min(64, a.ent_off[e + 1] - tb);
    const bool active = wave * 16 < nt;
    const int trow = wave * 16 + r; const bool tv = trow < nt;
    const int tc = min(trow, nt - 1);
    auto dof = [&](int i) { return 16 * (i >> 2) + 4 * kq + (i & 3); };      // reduction step i of lane group kq
    const float* fz = a.gz + (size_t)tb * a.gz_ld + (size_t)h * dim;
    const float* kz = a.ksrc + (size_t)tb * a.src_ld + (size_t)h * dim; const float* qz = a.qsrc + (size_t)tb * a.src_ld + (size_t)h * dim;
    const float* vz = a.vsrc + (size_t)tb * a.src_ld + (size_t)h * vdim;
    for (int i = tid; i < 4 * dimp; i += 256) {
        const int m = i / dimp, d = i - m * dimp;
        const float v = (d < dim && 16 * m < nt) ? fz[(size_t)min(16 * m + 15, nt - 1) * a.gz_ld + d] : 0.0f;
        tot[i] = v; et[i] = expf(v);
    }
    __syncthreads();
    for (int i = tid; i < 64 * dimp; i += 256) {
        const int s = i / dimp, d = i - s * dimp;
        kd[s * LK + d] = (s < nt && d < dim) ? kz[(size_t)s * a.src_ld + d] * expf(tot[(s >> 4) * dimp + d] - fz[(size_t)s * a.gz_ld + d]) : 0.0f;
    }
    float bonus = 0.0f, big = 0.0f;
    for (int i = 0; i < dq; i++) {
        const int d = dof(i);
        float q = 0.0f;
        if (active && d < dim) {
            const float x = qz[(size_t)tc * a.src_ld + d] * a.q_scale;
            float ev = 0.0f;
            if constexpr (WKV) { if (r > 0) ev = fz[(size_t)(tc - (trow < nt)) * a.gz_ld + d]; bonus = __builtin_fmaf(x * a.bonus[(size_t)h * dim + d], kz[(size_t)tc * a.src_ld + d], bonus); }
            else ev = fz[(size_t)tc * a.gz_ld + d];
            q = x * expf(ev);
            big = fmaxf(big, -tot[wave * dimp + d]);
        }
        qs[i * 64 + lane] = q;
    }
    if constexpr (WKV) { bonus += __shfl_xor(bonus, 16); bonus += __shfl_xor(bonus, 32); }
    big = fmaxf(big, __shfl_xor(big, 16)); big = fmaxf(big, __shfl_xor(big, 32));      // the same in every lane of a wave: lanes of one group share their channels
    __syncthreads();
    ln_f4 acc[DB];
#pragma unroll
    for (int c = 0; c < DB; c++) acc[c] = ln_f4{0.0f, 0.0f, 0.0f, 0.0f};
    if (active) {
#pragma nounroll
        for (int j = wave; j >= 0; j--) {
            ln_f4 st = ln_f4{0.0f, 0.0f, 0.0f, 0.0f};
            const float* krow = kd + (16 * j + r) * LK + 4 * kq;
            const float* ep = et + j * dimp + 4 * kq;
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
                for (int i0 = 0; i0 < dq; i0 += 4) {
                    const float4 k4 = *reinterpret_cast<const float4*>(krow + 4 * i0), e4 = *reinterpret_cast<const float4*>(ep + 4 * i0);
                    float q4[4];
#pragma unroll
                    for (int u = 0; u < 4; u++) q4[u] = qs[(i0 + u) * 64 + lane];
                    const float x0 = j == wave ? 1.0f / e4.x : 1.0f, x1 = j == wave ? 1.0f / e4.y : 1.0f, x2 = j == wave ? 1.0f / e4.z : 1.0f, x3 = j == wave ? 1.0f / e4.w : 1.0f;
                    st = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.x, q4[0] * x0, st, 0, 0, 0); st = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.y, q4[1] * x1, st, 0, 0, 0);
                    st = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.z, q4[2] * x2, st, 0, 0, 0); st = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.w, q4[3] * x3, st, 0, 0, 0);
                    if (j < wave) {          // on to the sub-block before: the queries take this one's decay along
                        qs[i0 * 64 + lane] = q4[0] * e4.x; qs[(i0 + 1) * 64 + lane] = q4[1] * e4.y; qs[(i0 + 2) * 64 + lane] = q4[2] * e4.z; qs[(i0 + 3) * 64 + lane] = q4[3] * e4.w;
                    }
                }
            }
            size_t srow[4];
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int s = 16 * j + 4 * kq + i;
                srow[i] = (size_t)min(s, nt - 1) * a.src_ld;
                if (j == wave) { if (WKV && s == trow) st[i] = bonus; else if (s > trow) st[i] = 0.0f; }
                if (!tv) st[i] = 0.0f;
            }
            float vf[4][DB];
#pragma unroll
            for (int i = 0; i < 4; i++)
#pragma unroll
                for (int c = 0; c < DB; c++) { const int cc = c * 16 + r; vf[i][c] = cc < vdim ? vz[srow[i] + cc] : 0.0f; }
#pragma unroll
            for (int i = 0; i < 4; i++)
#pragma unroll
                for (int c = 0; c < DB; c++) acc[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(vf[i][c], st[i], acc[c], 0, 0, 0);
        }
    }
    const float* Sc = a.sbuf + ((size_t)gc * H + h) * dim * vdim;
    for (int p0 = 0; p0 < dim; p0 += 32) {          // the state's share: passes over 32 of its rows
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
#pragma unroll 2
            for (int i = 0; i < 8; i++) {
                const int lr = dof(i);
                const float qi = lr < rows ? qs[(p0 / 4 + i) * 64 + lane] : 0.0f;
                const float* srow = sl + min(lr, rows - 1) * LS + r;
#pragma unroll
                for (int c = 0; c < DB; c++) acc[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(c * 16 + r < vdim ? srow[c * 16] : 0.0f, qi, acc[c], 0, 0, 0);
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
// (wave w: key rows 16 w .. and 16 (w + 4) ..).  S lives in the accumulators and, as the next block's operand, in LDS; the operands of the next block are requested
// before the current one is worked on.  Leaves S at the block's start in a.sbuf and U in place of v; the outputs are sv_lin_cout_kernel's.
template <int DT>          // 16-row tiles of a head's keys: 4 or 8
__global__ void __launch_bounds__(256) ln_delta_state_kernel(const KrSvLin a) {
    constexpr int DP = DT * 16, NW = DT / 4, LS = 20;      // NW key-row tiles per wave; LDS rows of 16 columns, 20 floats apart
    __shared__ __attribute__((aligned(16))) float Sl[DP * LS], Ul[64 * LS];
    const int e = blockIdx.x, h = blockIdx.y, cb = blockIdx.z, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, kq = lane >> 4;
    const int H = a.heads, dim = a.dim, vdim = a.vdim, hq = h / a.qk_group, col = cb * 16 + r; const bool cv = col < vdim; const int colc = cv ? col : 0;
    const int t0 = a.ent_off[e], t1 = a.ent_off[e + 1], nch = (t1 - t0 + 63) / 64, c0 = a.ent_chunk0[e];
    const bool fresh = a.pos[t0] == 0;
    float* Sg = a.state + (size_t)a.ent_slot[e] * a.state_stride + ((size_t)h * vdim + colc) * dim;
    ln_f4 S[NW];
#pragma unroll
    for (int n = 0; n < NW; n++)
#pragma unroll
        for (int i = 0; i < 4; i++) { const int d = (wave + 4 * n) * 16 + 4 * kq + i; S[n][i] = (!fresh && cv && d < dim) ? Sg[d] : 0.0f; }
    float y[2][DP / 4], kk[2][NW][16], xv[2][4], fs[2][4], fl[2];
    auto fetch = [&](int b, int c) {
        const int tb = t0 + 64 * c, nt = min(64, t1 - tb);
        const float* yp = a.aux + (size_t)(tb + min(16 * wave + r, nt - 1)) * H * dim + (size_t)h * dim;
#pragma unroll
        for (int i = 0; i < DP / 4; i++) { const int d = 16 * (i >> 2) + 4 * kq + (i & 3); y[b][i] = d < dim ? yp[d] : 0.0f; }
        const float* kp = a.ksrc + (size_t)tb * a.src_ld + (size_t)hq * dim;
#pragma unroll
        for (int n = 0; n < NW; n++) {
            const int d = (wave + 4 * n) * 16 + r;
#pragma unroll
            for (int j = 0; j < 16; j++) kk[b][n][j] = d < dim ? kp[(size_t)min(4 * j + kq, nt - 1) * a.src_ld + d] : 0.0f;
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
                const int d = (wave + 4 * n) * 16 + 4 * kq + i;
                Sl[d * LS + r] = S[n][i];
                if (cv && d < dim) sb[(size_t)d * vdim] = S[n][i];
            }
        __syncthreads();
        ln_f4 u = ln_f4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int i = 0; i < DP / 4; i++) u = __builtin_amdgcn_mfma_f32_16x16x4f32(y[b][i], Sl[(16 * (i >> 2) + 4 * kq + (i & 3)) * LS + r], u, 0, 0, 0);
        float* up = const_cast<float*>(a.vsrc) + (size_t)tb * a.src_ld + (size_t)h * vdim + col;
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int s = 16 * wave + 4 * kq + i; const bool ok = s < nt && cv;
            const float v = ok ? xv[b][i] - u[i] : 0.0f;
            Ul[s * LS + r] = v * expf(fl[b] - fs[b][i]);
            if (ok) up[(size_t)s * a.src_ld] = v;
        }
        __syncthreads();
        const float dec = expf(fl[b]);
#pragma unroll
        for (int n = 0; n < NW; n++) S[n] *= dec;
#pragma unroll
        for (int j = 0; j < 16; j++) {
            const float uu = Ul[(4 * j + kq) * LS + r];
#pragma unroll
            for (int n = 0; n < NW; n++) S[n] = __builtin_amdgcn_mfma_f32_16x16x4f32(kk[b][n][j], uu, S[n], 0, 0, 0);
        }
    };
    fetch(0, 0);
    for (int c = 0; c < nch; c += 2) {
        if (c + 1 < nch) fetch(1, c + 1);
        block(0, c);
        if (c + 2 < nch) fetch(0, c + 2);
        if (c + 1 < nch) block(1, c + 1);
    }
#pragma unroll
    for (int n = 0; n < NW; n++)
#pragma unroll
        for (int i = 0; i < 4; i++) { const int d = (wave + 4 * n) * 16 + 4 * kq + i; if (cv && d < dim) Sg[d] = S[n][i]; }
}
}  // namespace

bool kr_sv_lin_blocks_fit(int dim, int vdim) { return dim <= 128 && vdim <= 128; }
void kr_sv_lin_chan_blocks(const KrSvLin& a, hipStream_t st) {
    if (a.T <= 0 || a.n_entries <= 0 || a.n_chunks <= 0) return;
    const dim3 g(a.n_chunks, a.heads);
    const int dimp = ((a.dim + 15) / 16) * 16;
#define LN_LDS(K_, B_) do { if ((B_) > 48 * 1024) (void)hipFuncSetAttribute((const void*)K_, hipFuncAttributeMaxDynamicSharedMemorySize, (int)(B_)); } while (0)
    if (a.dim <= 64) { const size_t b = (size_t)(64 * 80 + 4 * 64) * 4; hipLaunchKernelGGL(ln_chan_local_kernel<4>, g, dim3(256), b, st, a); }
    else { const size_t b = (size_t)(64 * 144 + 4 * 128) * 4; LN_LDS(ln_chan_local_kernel<8>, b); hipLaunchKernelGGL(ln_chan_local_kernel<8>, g, dim3(256), b, st, a); }
    hipLaunchKernelGGL(ln_chan_scan_kernel, dim3(a.n_entries, a.heads, (a.dim * a.vdim + 255) / 256), dim3(256), 0, st, a);
    const size_t lds = ((size_t)64 * (dimp + 4) + 8 * dimp + 32 * (((a.vdim + 31) / 32) * 32 + 16) + (size_t)4 * (dimp / 4) * 64) * 4;
#define LN_CO(DB_, W_) do { LN_LDS((ln_chan_out_kernel<DB_, W_>), lds); hipLaunchKernelGGL((ln_chan_out_kernel<DB_, W_>), g, dim3(256), lds, st, a); } while (0)
    if (a.vdim <= 64) { if (a.kind == 7) LN_CO(4, true); else LN_CO(4, false); } else { if (a.kind == 7) LN_CO(8, true); else LN_CO(8, false); }
#undef LN_CO
}
void kr_sv_delta_blocks(const KrSvLin& a, hipStream_t st) {
    if (a.T <= 0 || a.n_entries <= 0 || a.n_chunks <= 0) return;
    const size_t lds = ((size_t)64 * (((a.dim + 15) / 16) * 16 + 4) + 2 * 64 * 68 + 128) * 4;
    LN_LDS(ln_delta_solve_kernel, lds);
    hipLaunchKernelGGL(ln_delta_solve_kernel, dim3(a.n_chunks, a.heads), dim3(256), lds, st, a);
    const dim3 gs(a.n_entries, a.heads, (a.vdim + 15) / 16);
    if (a.dim <= 64) hipLaunchKernelGGL(ln_delta_state_kernel<4>, gs, dim3(256), 0, st, a);
    else hipLaunchKernelGGL(ln_delta_state_kernel<8>, gs, dim3(256), 0, st, a);
    kr_sv_lin_block_out(a, st);
}

void kr_sv_shift(const KrSvShift& a, bool f32, hipStream_t st) {
    if (a.T <= 0) return;
    const dim3 grid(a.T, (a.width + 255) / 256);
    if (f32) hipLaunchKernelGGL(ln_shift_kernel<float>, grid, dim3(256), 0, st, a, (float*)a.out);
    else hipLaunchKernelGGL(ln_shift_kernel<uint16_t>, grid, dim3(256), 0, st, a, (uint16_t*)a.out);
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
    hipLaunchKernelGGL(ln_delta_prep_kernel, dim3(a.T, 2 * a.kv_heads + a.heads), dim3(64), 0, st, a);
    const int C = 2 * a.kv_heads * a.dim + a.heads * a.vdim;
    if (!a.single && a.taps > 1) hipLaunchKernelGGL(ln_delta_save_kernel, dim3(a.n_entries, a.taps - 1, (C + 255) / 256), dim3(256), 0, st, a);
}
void kr_sv_lt_prep(float* z, int ld, int cols, const float* decay, int heads, float4* tok, int T, hipStream_t st) {
    if (T <= 0) return;
    const int n = cols > heads ? cols : heads;
    hipLaunchKernelGGL(ln_lt_prep_kernel, dim3(T, (n + 255) / 256), dim3(256), 0, st, z, ld, cols, decay, heads, tok);
}
void kr_sv_row_out(const float* o, int n, const float* w, const float* gate, int gate_ld, float eps, float scale, void* out, int out_ld, bool f32, int T, hipStream_t st) {
    if (T <= 0) return;
    if (f32) hipLaunchKernelGGL(ln_row_out_kernel<float>, dim3(T), dim3(256), 0, st, o, n, w, gate, gate_ld, eps, scale, (float*)out, out_ld);
    else hipLaunchKernelGGL(ln_row_out_kernel<uint16_t>, dim3(T), dim3(256), 0, st, o, n, w, gate, gate_ld, eps, scale, (uint16_t*)out, out_ld);
}
