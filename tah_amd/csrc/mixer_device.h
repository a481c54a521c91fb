// Device-side helpers of the layer mechanisms in row_norm.hip, delta_rule.hip, latent_attn.hip, window_attn.hip and moe.hip.
#pragma once
#include "duo_device.h"
#include "tah_mixers.h"

namespace tah {

typedef __attribute__((__vector_size__(8 * sizeof(float)))) float f32x8;

// Eight elements of a row as float32.
__device__ __forceinline__ void load8(const __bf16* p, float (&v)[8]) {
    const bf16x8 x = *reinterpret_cast<const bf16x8*>(p);
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = (float)x[i];
}
__device__ __forceinline__ void load8(const float* p, float (&v)[8]) {
    const f32x4 a = *reinterpret_cast<const f32x4*>(p), b = *reinterpret_cast<const f32x4*>(p + 4);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        v[i] = a[i];
        v[4 + i] = b[i];
    }
}
__device__ __forceinline__ bf16x8 to_bf16x8(const float (&v)[8]) {
    bf16x8 x;
#pragma unroll
    for (int i = 0; i < 8; ++i) x[i] = (__bf16)v[i];
    return x;
}
__device__ __forceinline__ void store8(__bf16* p, const float (&v)[8]) { *reinterpret_cast<bf16x8*>(p) = to_bf16x8(v); }
__device__ __forceinline__ void store8(float* p, const float (&v)[8]) {
    *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
    *reinterpret_cast<f32x4*>(p + 4) = f32x4{v[4], v[5], v[6], v[7]};
}

// 16-byte unit of the rows form of tah_linear_rows that holds row r, columns c ... c + 7 (c % 8 == 0)
__device__ __host__ __forceinline__ int64_t rows_form_unit(int r, int c) {
    return ((int64_t)(c / 32) * 2 + r / 16) * 64 + (r % 16) + 16 * ((c % 32) / 8);
}
// element of it
__device__ __host__ __forceinline__ int64_t rows_form_elem(int r, int c) { return rows_form_unit(r, c) * 8 + c % 8; }

__device__ __forceinline__ float wave_sum(float x) {
#pragma unroll
    for (int m = 32; m >= 1; m >>= 1) x += __shfl_xor(x, m);
    return x;
}
__device__ __forceinline__ float wave_max(float x) {
#pragma unroll
    for (int m = 32; m >= 1; m >>= 1) x = fmaxf(x, __shfl_xor(x, m));
    return x;
}
// Sum over a workgroup of kWaves waves; `red` is LDS of kWaves floats that nobody else is using.
template <int kWaves>
__device__ __forceinline__ float block_sum(float x, float* red) {
    x = wave_sum(x);
    if (threadIdx.x % kWave == 0) red[threadIdx.x / kWave] = x;
    __syncthreads();
    float s = 0.f;
#pragma unroll
    for (int w = 0; w < kWaves; ++w) s += red[w];
    __syncthreads();
    return s;
}

// Accurate forms: what enters a recurrence, a norm or a router is float32 to the last bits.
__device__ __forceinline__ float sigmoid_exact(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float silu_exact(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float softplus_exact(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
__device__ __forceinline__ float gelu_tanh_exact(float x) {
    return 0.5f * x * (1.0f + tanhf(0.7978845608028654f * (x + 0.044715f * x * x * x)));
}

// x > 0: a x^2 + x / 2, else b (exp(x) - 1 - x) + x / 2
__device__ __forceinline__ float xielu(float x, float a, float b) { return (x > 0.f ? a * x * x : b * (expm1f(x) - x)) + 0.5f * x; }
// gate cut off above the limit, up on both sides of it: g sigmoid(slope g) (u + 1)
__device__ __forceinline__ float clamped_gate(float g, float u, float limit, float slope) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g / (1.0f + fast_exp2(-slope * kLog2e * g)) * (u + 1.0f);
}
__device__ __forceinline__ float clamped_gate_exact(float g, float u, float limit, float slope) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g / (1.0f + expf(-slope * g)) * (u + 1.0f);
}

// ---- attention on the matrix cores ----
// Which of a SIMD's waves is served first from here on (within the kernel)
#ifdef TAH_CPU_EMU
#define TAH_WAVE_PRIORITY(n)
#else
#define TAH_WAVE_PRIORITY(n) __builtin_amdgcn_s_setprio(n)
#endif
constexpr float kNoScore = -1e30f;  // below every score, and finite: differences of it are numbers

__device__ __forceinline__ f32x4 mfma16(bf16x8 a, bf16x8 b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }
__device__ __forceinline__ bf16x8 join8(bf16x4 lo, bf16x4 hi) { return __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7); }
__device__ __forceinline__ bf16x4 to_bf16x4(const float (&w)[4]) { return __builtin_convertvector((f32x4{w[0], w[1], w[2], w[3]}), bf16x4); }
// Eight numbers as two bf16 terms each, the leading bits and what they leave: sixteen bits of them together.
__device__ __forceinline__ void split_bf16x8(const float (&w)[8], bf16x8& hi, bf16x8& lo) {
    uint32_t h[4];
    float rest[8];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const uint32_t a = __float_as_uint(w[2 * i]), b = __float_as_uint(w[2 * i + 1]) & 0xffff0000u;
        h[i] = (a >> 16) | b;
        rest[2 * i] = w[2 * i] - __uint_as_float(a & 0xffff0000u);
        rest[2 * i + 1] = w[2 * i + 1] - __uint_as_float(b);
    }
    __builtin_memcpy(&hi, h, 16);
    lo = __builtin_convertvector((f32x8{rest[0], rest[1], rest[2], rest[3], rest[4], rest[5], rest[6], rest[7]}), bf16x8);
}
// The larger of two scores (finite or -inf), in one instruction: fmaxf has to quieten NaNs of operands it knows nothing about.
__device__ __forceinline__ float score_max(float a, float b) {
#ifdef TAH_CPU_EMU
    return fmaxf(a, b);
#else
    return __builtin_amdgcn_fmed3f(a, b, 3.0e38f);
#endif
}
// x over the four lane groups that share l % 16
__device__ __forceinline__ float groups_max(float x) {
    x = fmaxf(x, __shfl_xor(x, 16));
    return fmaxf(x, __shfl_xor(x, 32));
}
__device__ __forceinline__ float groups_sum(float x) {
    x += __shfl_xor(x, 16);
    return x + __shfl_xor(x, 32);
}

inline bool aligned_16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }
inline int launch_status() { return hipGetLastError() == hipSuccess ? TAH_OK : TAH_E_LAUNCH; }

}  // namespace tah
