// kr_serve_rglru.hip -- the real-gated linear recurrence of the serving store (KrSvRglru, gfx950, wave64).
//
// Portions: a chunk is 64 tokens of one request.  sv_rglru_gate_kernel, a workgroup per (chunk, 128 channels of a block): the convolution feeds both gate
// products from LDS, the lane that holds a channel's gates of 16 tokens in its accumulators forms decay and input there and walks them, and four lanes
// compose to the chunk: it leaves per token (product of the decays, state from zero) since the chunk's start.  sv_rglru_chain_kernel carries S over the
// chunks, sv_rglru_out_kernel forms S of every token from its chunk's start, gates it and keeps the convolution's last rows.
// Decode: sv_rglru_step_kernel does all of it for one token per request in one launch.
#include <hip/hip_runtime.h>
#include <math.h>
#include <stdint.h>

#include "kr_device.h"
#include "kr_serve_ops.h"

namespace {
typedef float rg_f4 __attribute__((ext_vector_type(4)));
typedef __bf16 rg_b8 __attribute__((ext_vector_type(8)));
typedef uint32_t rg_u4 __attribute__((ext_vector_type(4)));
typedef uint32_t rg_u2 __attribute__((ext_vector_type(2)));

__device__ __forceinline__ float rg_ld(const float* p) { return *p; }
__device__ __forceinline__ float rg_ld(const uint16_t* p) { return kr_bf16_to_f32(*p); }
// sigmoid on the hardware's exponential and reciprocal (one unit in the last place each)
__device__ __forceinline__ float rg_sigmoid(float z) { return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z)); }
// tanh form of gelu: (1 + tanh w) / 2 = sigmoid(2 w)
__device__ __forceinline__ float rg_gelu(float z) { return z * rg_sigmoid(2.0f * 0.7978845608028654f * (z + 0.044715f * z * z * z)); }
// decay d = exp(x) and input sqrt(1 - d^2) i u of one token and channel from the gates' logits.  Near one d and 1 - d^2 both come from m = exp(x) - 1 as a
// polynomial in x (terms to x^6: 5e-8 of m at x = -1/4), so neither loses digits; below, from the exponential itself
__device__ __forceinline__ void rg_decay_input(float zr, float zi, float rate, float u, float& d, float& b) {
    const float x = rate * rg_sigmoid(zr);
    float p = __builtin_fmaf(x, 1.0f / 720.0f, 1.0f / 120.0f);
    p = __builtin_fmaf(x, p, 1.0f / 24.0f); p = __builtin_fmaf(x, p, 1.0f / 6.0f); p = __builtin_fmaf(x, p, 0.5f);
    const float m = __builtin_fmaf(x * x, p, x), e = __builtin_amdgcn_exp2f(1.4426950408889634f * x);
    const bool near1 = x > -0.25f;
    d = near1 ? 1.0f + m : e;
    const float q = near1 ? -m * (2.0f + m) : __builtin_fmaf(-e, e, 1.0f);
    b = __builtin_amdgcn_sqrtf(q) * rg_sigmoid(zi) * u;
}
// two floats as two bf16 (round to nearest even), the first in the low half
__device__ __forceinline__ uint32_t rg_pack2(float lo, float hi) {
    typedef __bf16 b2 __attribute__((ext_vector_type(2)));
    b2 v; v[0] = (__bf16)lo; v[1] = (__bf16)hi;
    return __builtin_bit_cast(uint32_t, v);
}

struct RgChunk { int e, t0, n, row0, p0, slot; };      // entry, first token, tokens, first row and first position of the entry's portion
__device__ __forceinline__ RgChunk rg_chunk(const KrSvRglru& a, int ck) {
    RgChunk c;
    c.e = 0;
    while (c.e + 1 < a.n_entries && ck >= a.ent_chunk0[c.e + 1]) c.e++;
    c.row0 = a.ent_off[c.e];
    c.t0 = c.row0 + (ck - a.ent_chunk0[c.e]) * 64;
    c.n = min(64, a.ent_off[c.e + 1] - c.t0);
    c.p0 = a.pos[c.row0]; c.slot = a.ent_slot[c.e];
    return c;
}
// the convolution's input of channel c, j rows after the chunk's first token (j may be negative)
__device__ __forceinline__ float rg_x(const KrSvRglru& a, const RgChunk& k, int j, int c, float xb) {
    const int t = k.t0 + j;
    if (j >= k.n) return 0.0f;
    if (t >= k.row0) return a.x[(size_t)t * a.ld + c] + xb;
    const int p = k.p0 + (t - k.row0);
    return p < 0 ? 0.0f : a.ring[((size_t)k.slot * a.taps + p % a.taps) * a.width + c];
}

#define RG_CH 128      // channels of a workgroup, and of a slab of the reduction
#define RG_LDU 136     // LDS row of RG_CH bf16 (+ 8): 16-byte fragment reads stay aligned and consecutive rows start 4 banks apart
#define RG_LDF 132     // the same of RG_CH floats
// Token 16 a + 4 m + i of a chunk lies in LDS row 16 m + 4 a + i: product m's rows then are token 16 (r / 4) + 4 m + r % 4 for row r -- so that a lane's
// accumulators are 16 consecutive tokens -- and its fragment reads are 16 consecutive LDS rows, which fall into distinct banks
__device__ __forceinline__ int rg_row(int t) { return 16 * ((t >> 2) & 3) + 4 * (t >> 4) + (t & 3); }
// TAPS: the convolution's taps when known, 0 = any number
template <typename T, int TAPS>
__global__ void __launch_bounds__(512) __attribute__((amdgpu_waves_per_eu(sizeof(T) == 2 ? 4 : 2))) sv_rglru_gate_kernel(const KrSvRglru a) {
    constexpr bool BF = sizeof(T) == 2;
    constexpr int VEC = 16 / sizeof(T);
    // bf16 store: u as three bf16 terms (8 mantissa bits each: their sum is u); f32 store: u itself
    __shared__ __attribute__((aligned(16))) char lds[BF ? 3 * 64 * RG_LDU * 2 : 64 * RG_LDF * 4];
    uint16_t* up = (uint16_t*)lds; float* uf = (float*)lds;
    const int size = a.width / a.blocks, nsl = (size + RG_CH - 1) / RG_CH;
    const int b = blockIdx.y / nsl, ns = blockIdx.y % nsl;
    const RgChunk k = rg_chunk(a, blockIdx.x);
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r15 = lane & 15, qd = lane >> 4;
    const int cl = ns * RG_CH + wave * 16 + r15;                // the lane's channel within the block
    const bool live = cl < size;
    const int c = b * size + min(cl, size - 1);
    const T* gw = (const T*)a.gw + (size_t)b * 2 * size * size;
    const T* wr[2] = {gw + (size_t)min(cl, size - 1) * size, gw + (size_t)(size + min(cl, size - 1)) * size};
    const bool vec = size % VEC == 0 && (uintptr_t)a.gw % 16 == 0;
    rg_f4 acc[2][4];
#pragma unroll
    for (int g = 0; g < 2; g++)
#pragma unroll
        for (int m = 0; m < 4; m++) acc[g][m] = rg_f4{0.0f, 0.0f, 0.0f, 0.0f};
    // the slabs of the block in turn, this workgroup's own channels last: their u stays in LDS for the recurrence
    for (int s = 1; s <= nsl; s++) {
        const int k0 = (ns + s) % nsl * RG_CH;
        // ---- u of the slab: a thread forms 8 consecutive tokens of two channels
        const int kc = k0 + 2 * lane, j0 = wave * 8, cc = b * size + kc;
        float u[8][2];
#pragma unroll
        for (int j = 0; j < 8; j++) u[j][0] = u[j][1] = 0.0f;
        bool done = kc >= size;
        if constexpr (TAPS > 0) {
            if (!done && kc + 1 < size && k.t0 + j0 - (TAPS - 1) >= k.row0 && j0 + 8 <= k.n) {      // both channels exist and every row is one of this step's
                const float* xp = a.x + (size_t)(k.t0 + j0 - (TAPS - 1)) * a.ld + cc;
                float xs[7 + TAPS][2], wt[2][TAPS];
#pragma unroll
                for (int i = 0; i < 7 + TAPS; i++) __builtin_memcpy(xs[i], xp + (size_t)i * a.ld, 8);
#pragma unroll
                for (int q = 0; q < 2; q++) {
                    const float xb = a.x_b[cc + q], cb = a.conv_b[cc + q];
#pragma unroll
                    for (int i = 0; i < TAPS; i++) wt[q][i] = a.conv[(size_t)(cc + q) * TAPS + i];
#pragma unroll
                    for (int i = 0; i < 7 + TAPS; i++) xs[i][q] += xb;
#pragma unroll
                    for (int j = 0; j < 8; j++) {
                        float v = cb;
#pragma unroll
                        for (int i = 0; i < TAPS; i++) v = __builtin_fmaf(wt[q][i], xs[j + i][q], v);
                        u[j][q] = v;
                    }
                }
                done = true;
            }
        }
        if (!done) {
#pragma unroll
            for (int q = 0; q < 2; q++) {
                if (kc + q >= size) continue;
                const float xb = a.x_b[cc + q], cb = a.conv_b[cc + q];
#pragma unroll
                for (int j = 0; j < 8; j++) u[j][q] = cb;
                for (int i = 0; i < a.taps; i++) {
                    const float wt = a.conv[(size_t)(cc + q) * a.taps + i];
#pragma unroll
                    for (int j = 0; j < 8; j++) u[j][q] = __builtin_fmaf(wt, rg_x(a, k, j0 + j - (a.taps - 1) + i, cc + q, xb), u[j][q]);
                }
            }
        }
        // ---- weights of the slab: 16-byte pieces in the order the products take them
        constexpr int NP = BF ? 4 : 8;
        rg_u4 wv[2][NP];
#pragma unroll
        for (int g = 0; g < 2; g++)
#pragma unroll
            for (int q = 0; q < NP; q++) {
                const int kk = k0 + (BF ? q * 32 + 8 * qd : 32 * qd + 4 * q);
                rg_u4 v = {0u, 0u, 0u, 0u};
                if (vec) { if (kk < size) v = *reinterpret_cast<const rg_u4*>(wr[g] + kk); }
                else {
#pragma unroll
                    for (int i = 0; i < VEC; i++) if (kk + i < size) {
                        if constexpr (BF) v[i >> 1] |= (uint32_t)((const uint16_t*)wr[g])[kk + i] << (16 * (i & 1));
                        else v[i] = __float_as_uint(((const float*)wr[g])[kk + i]);
                    }
                }
                wv[g][q] = v;
            }
        __syncthreads();                                        // the previous slab's products have read LDS
#pragma unroll
        for (int j = 0; j < 8; j++) {
            const int t = rg_row(j0 + j);
            if constexpr (BF) {
                float r0 = u[j][0], r1 = u[j][1];
#pragma unroll
                for (int pl = 0; pl < 3; pl++) {
                    const uint32_t h = rg_pack2(r0, r1);
                    *reinterpret_cast<uint32_t*>(&up[(pl * 64 + t) * RG_LDU + 2 * lane]) = h;
                    r0 -= __uint_as_float(h << 16); r1 -= __uint_as_float(h & 0xFFFF0000u);
                }
            } else *reinterpret_cast<float2*>(&uf[t * RG_LDF + 2 * lane]) = make_float2(u[j][0], u[j][1]);
        }
        __syncthreads();
        // ---- both gates' logits
        if constexpr (BF) {
#pragma unroll
            for (int q = 0; q < 4; q++)
#pragma unroll
                for (int pl = 2; pl >= 0; pl--)                 // small terms first
#pragma unroll
                    for (int m = 0; m < 4; m++) {
                        const rg_b8 av = __builtin_bit_cast(rg_b8, *reinterpret_cast<const rg_u4*>(&up[(pl * 64 + 16 * m + r15) * RG_LDU + q * 32 + 8 * qd]));
#pragma unroll
                        for (int g = 0; g < 2; g++) acc[g][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(av, __builtin_bit_cast(rg_b8, wv[g][q]), acc[g][m], 0, 0, 0);
                    }
        } else {
#pragma unroll
            for (int q = 0; q < 8; q++)
#pragma unroll
                for (int m = 0; m < 4; m++) {
                    const float4 av = *reinterpret_cast<const float4*>(&uf[(16 * m + r15) * RG_LDF + 32 * qd + 4 * q]);
                    const float af[4] = {av.x, av.y, av.z, av.w};
#pragma unroll
                    for (int i = 0; i < 4; i++)
#pragma unroll
                        for (int g = 0; g < 2; g++) acc[g][m] = __builtin_amdgcn_mfma_f32_16x16x4f32(af[i], __uint_as_float(wv[g][q][i]), acc[g][m], 0, 0, 0);
                }
        }
    }
    // ---- the lane's 16 tokens [16 qd, 16 qd + 16) of channel c: decay and input, walked from zero
    const float br = a.gb[c], bi = a.gb[a.width + c], rate = a.rate[c];
    float A[16], H[16], ca = 1.0f, ch = 0.0f;
#pragma unroll
    for (int j = 0; j < 16; j++) {
        const int t = 16 * qd + j, tr = rg_row(t), ul = wave * 16 + r15;
        const float u = BF ? kr_bf16_to_f32(up[tr * RG_LDU + ul]) + (kr_bf16_to_f32(up[(64 + tr) * RG_LDU + ul]) + kr_bf16_to_f32(up[(128 + tr) * RG_LDU + ul])) : uf[tr * RG_LDF + ul];
        float d, in;
        rg_decay_input(acc[0][j >> 2][j & 3] + br, acc[1][j >> 2][j & 3] + bi, rate, u, d, in);
        if (t >= k.n) { d = 1.0f; in = 0.0f; }                  // rows past the portion
        ca *= d; ch = __builtin_fmaf(d, ch, in);
        A[j] = ca; H[j] = ch;
    }
    // ---- the lanes 16 apart hold the earlier and later tokens of the channel
    float pa = 1.0f, ph = 0.0f;                                  // composition of the lanes before this one
#pragma unroll
    for (int q = 0; q < 3; q++) {
        const float qa = __shfl(ca, r15 + 16 * q), qh = __shfl(ch, r15 + 16 * q);
        if (q < qd) { ph = __builtin_fmaf(qa, ph, qh); pa *= qa; }
    }
    if (!live) return;
#pragma unroll
    for (int j = 0; j < 16; j++) {
        const int t = 16 * qd + j;
        if (t < k.n) a.ab[(size_t)(k.t0 + t) * a.width + c] = make_float2(A[j] * pa, __builtin_fmaf(A[j], ph, H[j]));
    }
    if (qd == 3) a.agg[(size_t)blockIdx.x * a.width + c] = make_float2(ca * pa, __builtin_fmaf(ca, ph, ch));
}

// S at the start of every chunk of an entry and, after the last one, the request's state: a thread per channel
__global__ void __launch_bounds__(64) sv_rglru_chain_kernel(const KrSvRglru a) {
    const int c = blockIdx.x * 64 + threadIdx.x, e = blockIdx.y;
    if (c >= a.width) return;
    const int c0 = a.ent_chunk0[e], c1 = a.ent_chunk0[e + 1];
    float* st = a.state + (size_t)a.ent_slot[e] * a.width + c;
    float S = a.pos[a.ent_off[e]] > 0 ? *st : 0.0f;
    for (int k = c0; k < c1; k += 16) {
        float2 v[16];
#pragma unroll
        for (int i = 0; i < 16; i++) v[i] = k + i < c1 ? a.agg[(size_t)(k + i) * a.width + c] : make_float2(1.0f, 0.0f);
#pragma unroll
        for (int i = 0; i < 16; i++) {
            if (k + i < c1) a.start[(size_t)(k + i) * a.width + c] = S;
            S = __builtin_fmaf(v[i].x, S, v[i].y);
        }
    }
    *st = S;
}

// out = S * gelu_tanh(y + y_b); the portion's last taps - 1 convolution inputs go to the ring.  A workgroup per (chunk, 64 * V channels), 16 tokens per wave
template <typename T, int V>
__global__ void __launch_bounds__(256) sv_rglru_out_kernel(const KrSvRglru a) {
    const RgChunk k = rg_chunk(a, blockIdx.x);
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c = (blockIdx.y * 64 + lane) * V;
    if (c >= a.width) return;
    float S0[V], yb[V];
#pragma unroll
    for (int i = 0; i < V; i++) { S0[i] = a.start[(size_t)blockIdx.x * a.width + c + i]; yb[i] = a.y_b[c + i]; }
    const int last = a.ent_off[k.e + 1] - (a.taps - 1), t1 = k.t0 + min(k.n, (wave + 1) * 16);
#pragma unroll 4
    for (int t = k.t0 + wave * 16; t < t1; t++) {
        float y[V], A[V], H[V];
        const float* yp = a.y + (size_t)t * a.ld + c;
        const float2* ap = a.ab + (size_t)t * a.width + c;
        if constexpr (V == 4) {
            const float4 yv = *reinterpret_cast<const float4*>(yp), p = reinterpret_cast<const float4*>(ap)[0], q = reinterpret_cast<const float4*>(ap)[1];
            y[0] = yv.x; y[1] = yv.y; y[2] = yv.z; y[3] = yv.w;
            A[0] = p.x; H[0] = p.y; A[1] = p.z; H[1] = p.w; A[2] = q.x; H[2] = q.y; A[3] = q.z; H[3] = q.w;
        } else {
#pragma unroll
            for (int i = 0; i < V; i++) { y[i] = yp[i]; A[i] = ap[i].x; H[i] = ap[i].y; }
        }
        float o[V];
#pragma unroll
        for (int i = 0; i < V; i++) o[i] = __builtin_fmaf(A[i], S0[i], H[i]) * rg_gelu(y[i] + yb[i]);
        T* op = (T*)a.out + (size_t)t * a.out_ld + c;
        if constexpr (V == 4 && sizeof(T) == 2) {
            const rg_u2 w = {(uint32_t)kr_f32_to_bf16(o[0]) | ((uint32_t)kr_f32_to_bf16(o[1]) << 16), (uint32_t)kr_f32_to_bf16(o[2]) | ((uint32_t)kr_f32_to_bf16(o[3]) << 16)};
            *reinterpret_cast<rg_u2*>(op) = w;
        } else if constexpr (V == 4) {
            *reinterpret_cast<float4*>(op) = make_float4(o[0], o[1], o[2], o[3]);
        } else {
#pragma unroll
            for (int i = 0; i < V; i++) {
                if constexpr (sizeof(T) == 2) op[i] = kr_f32_to_bf16(o[i]); else op[i] = o[i];
            }
        }
        if (t >= last) {
            const int p = k.p0 + (t - k.row0);
#pragma unroll
            for (int i = 0; i < V; i++) a.ring[((size_t)k.slot * a.taps + p % a.taps) * a.width + c + i] = a.x[(size_t)t * a.ld + c + i] + a.x_b[c + i];
        }
    }
}

// One token per entry.  A workgroup per (MB entries, 4 CN channels of a block): u of the whole block in LDS, a wave multiplies it by both gates' rows of CN
// channels (lanes 0 .. 31 the first gate, 32 .. 63 the second), and the lanes that then hold a channel finish it.  The ring has one row more than the
// convolution looks back, so the row a workgroup writes is none that another one still reads.
template <typename T, int MB, int CN>
__global__ void __launch_bounds__(256) sv_rglru_step_kernel(const KrSvRglru a) {
    extern __shared__ float us[];            // [MB][size]
    constexpr int VEC = 16 / sizeof(T);
    const int size = a.width / a.blocks, nsl = (size + 4 * CN - 1) / (4 * CN), e0 = blockIdx.x * MB;
    const int b = blockIdx.y / nsl, c0 = ((blockIdx.y % nsl) * 4 + (threadIdx.x >> 6)) * CN;
    const int tid = threadIdx.x, lane = tid & 63, g = lane >> 5, l32 = lane & 31;
    const T* gw = (const T*)a.gw + ((size_t)b * 2 + g) * size * size;
    const bool vec = size % VEC == 0 && (uintptr_t)a.gw % 16 == 0;
    const T* wr[CN];
#pragma unroll
    for (int n = 0; n < CN; n++) wr[n] = gw + (size_t)min(c0 + n, size - 1) * size;
    rg_u4 wv[CN];
    if (vec) {
#pragma unroll
        for (int n = 0; n < CN; n++) wv[n] = *reinterpret_cast<const rg_u4*>(wr[n] + min(l32 * VEC, size - VEC));      // requested before the convolution
    }
    // what the finishing lane (entry fm, channel c0 + fn) needs besides the logits
    const int fm = min(lane / CN, MB - 1), fn = lane % CN, fe = min(e0 + fm, a.n_entries - 1);
    const bool fin = lane < CN * MB && e0 + lane / CN < a.n_entries && c0 + fn < size;
    const int fc = b * size + min(c0 + fn, size - 1), ft = a.ent_off[fe], fs = a.ent_slot[fe], fp = a.pos[ft];
    const float fy = a.y[(size_t)ft * a.ld + fc] + a.y_b[fc], fx = a.x[(size_t)ft * a.ld + fc] + a.x_b[fc], br = a.gb[fc], bi = a.gb[a.width + fc], rate = a.rate[fc];
    const float fS = fp > 0 ? a.state[(size_t)fs * a.width + fc] : 0.0f;
    for (int i = tid; i < MB * size; i += 256) {
        const int m = i / size, cc = b * size + (i - m * size), e = min(e0 + m, a.n_entries - 1), t = a.ent_off[e], p = a.pos[t], sl = a.ent_slot[e];
        const float* w = a.conv + (size_t)cc * a.taps;
        float v = a.conv_b[cc];
        for (int d = min(a.taps - 1, p); d > 0; d--) v = __builtin_fmaf(w[a.taps - 1 - d], a.ring[((size_t)sl * a.taps + (p - d) % a.taps) * a.width + cc], v);
        us[i] = __builtin_fmaf(w[a.taps - 1], a.x[(size_t)t * a.ld + cc] + a.x_b[cc], v);
    }
    __syncthreads();
    float acc[MB][CN];
#pragma unroll
    for (int m = 0; m < MB; m++)
#pragma unroll
        for (int n = 0; n < CN; n++) acc[m][n] = 0.0f;
    if (vec) {
        for (int k = l32 * VEC; k < size; k += 32 * VEC) {
            if (k >= 32 * VEC) {
#pragma unroll
                for (int n = 0; n < CN; n++) wv[n] = *reinterpret_cast<const rg_u4*>(wr[n] + k);
            }
#pragma unroll
            for (int i = 0; i < VEC; i++) {
                float w[CN];
#pragma unroll
                for (int n = 0; n < CN; n++) {
                    if constexpr (sizeof(T) == 2) w[n] = (i & 1) ? __uint_as_float(wv[n][i >> 1] & 0xFFFF0000u) : __uint_as_float(wv[n][i >> 1] << 16);
                    else w[n] = __uint_as_float(wv[n][i]);
                }
#pragma unroll
                for (int m = 0; m < MB; m++) {
                    const float u = us[m * size + k + i];
#pragma unroll
                    for (int n = 0; n < CN; n++) acc[m][n] = __builtin_fmaf(w[n], u, acc[m][n]);
                }
            }
        }
    } else {
        for (int k = l32; k < size; k += 32) {
#pragma unroll
            for (int n = 0; n < CN; n++) {
                const float w = rg_ld(wr[n] + k);
#pragma unroll
                for (int m = 0; m < MB; m++) acc[m][n] = __builtin_fmaf(w, us[m * size + k], acc[m][n]);
            }
        }
    }
    float zr = 0.0f, zi = 0.0f;
#pragma unroll
    for (int m = 0; m < MB; m++)
#pragma unroll
        for (int n = 0; n < CN; n++) {
            float v = acc[m][n];
#pragma unroll
            for (int o = 16; o > 0; o >>= 1) v += __shfl_xor(v, o);
            const float other = __shfl_xor(v, 32);
            if (lane == m * CN + n) { zr = v; zi = other; }       // lanes below 32: v is the first gate's
        }
    if (!fin) return;
    float d, in;
    rg_decay_input(zr + br, zi + bi, rate, us[fm * size + c0 + fn], d, in);
    const float S = __builtin_fmaf(d, fS, in), o = S * rg_gelu(fy);
    a.state[(size_t)fs * a.width + fc] = S;
    if (a.taps > 1) a.ring[((size_t)fs * a.taps + fp % a.taps) * a.width + fc] = fx;
    T* op = (T*)a.out + (size_t)ft * a.out_ld + fc;
    if constexpr (sizeof(T) == 2) *op = kr_f32_to_bf16(o); else *op = o;
}
}  // namespace

// the step kernel keeps a block's u of up to four entries in 64 KB of LDS
bool kr_sv_rglru_fits(int width, int blocks, int taps) {
    return width >= 1 && blocks >= 1 && width % blocks == 0 && width / blocks <= 4096 && taps >= 1 && taps <= 64;
}

void kr_sv_rglru_step(const KrSvRglru& a, bool f32, hipStream_t st) {
    if (a.n_entries <= 0) return;
    const int size = a.width / a.blocks, mb = a.n_entries == 1 ? 1 : 4;
    // channels per wave: four when that still gives every compute unit two workgroups, else two
    const int eg = (a.n_entries + mb - 1) / mb, cn = (long)eg * a.width / 16 >= 512 ? 4 : 2;
    const dim3 grid(eg, a.blocks * ((size + 4 * cn - 1) / (4 * cn)));
    const size_t lds = (size_t)mb * size * sizeof(float);
#define RG_S(T_, MB_) do { if (cn == 4) hipLaunchKernelGGL((sv_rglru_step_kernel<T_, MB_, 4>), grid, dim3(256), lds, st, a); \
                           else hipLaunchKernelGGL((sv_rglru_step_kernel<T_, MB_, 2>), grid, dim3(256), lds, st, a); } while (0)
    if (f32) { if (mb == 1) RG_S(float, 1); else RG_S(float, 4); }
    else { if (mb == 1) RG_S(uint16_t, 1); else RG_S(uint16_t, 4); }
#undef RG_S
}

void kr_sv_rglru_portions(const KrSvRglru& a, bool f32, hipStream_t st) {
    if (a.n_chunks <= 0) return;
    const int size = a.width / a.blocks;
    const dim3 grid(a.n_chunks, a.blocks * ((size + RG_CH - 1) / RG_CH));
#define RG_G(T_, N_) hipLaunchKernelGGL((sv_rglru_gate_kernel<T_, N_>), grid, dim3(512), 0, st, a)
    if (f32) { if (a.taps == 4) RG_G(float, 4); else RG_G(float, 0); }
    else { if (a.taps == 4) RG_G(uint16_t, 4); else RG_G(uint16_t, 0); }
#undef RG_G
    hipLaunchKernelGGL(sv_rglru_chain_kernel, dim3((a.width + 63) / 64, a.n_entries), dim3(64), 0, st, a);
    const bool v4 = a.width % 4 == 0 && a.ld % 4 == 0 && a.out_ld % 4 == 0 && (uintptr_t)a.y % 16 == 0 && (uintptr_t)a.out % 16 == 0 && (uintptr_t)a.ab % 16 == 0;
    const dim3 og(a.n_chunks, v4 ? (a.width / 4 + 63) / 64 : (a.width + 63) / 64);
    if (f32) { if (v4) hipLaunchKernelGGL((sv_rglru_out_kernel<float, 4>), og, dim3(256), 0, st, a); else hipLaunchKernelGGL((sv_rglru_out_kernel<float, 1>), og, dim3(256), 0, st, a); }
    else { if (v4) hipLaunchKernelGGL((sv_rglru_out_kernel<uint16_t, 4>), og, dim3(256), 0, st, a); else hipLaunchKernelGGL((sv_rglru_out_kernel<uint16_t, 1>), og, dim3(256), 0, st, a); }
}
