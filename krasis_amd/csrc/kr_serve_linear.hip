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
}  // namespace

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
