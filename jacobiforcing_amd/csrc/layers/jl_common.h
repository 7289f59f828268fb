// jl_common.h — shared by the translation units of libjf_layers.so (gfx950 / CDNA4 only): the layer kernels of the models whose
// forward is not stock PyTorch (32-bit residual stream, windowed attention with a distance bias and mixed heads, retention,
// routed experts).  Activations are float or bfloat16 (dtype code JL_F32 / JL_BF16); everything the kernels accumulate,
// normalise, exponentiate or carry from token to token is float.
#ifndef JL_COMMON_H
#define JL_COMMON_H

#include <hip/hip_runtime.h>
#include <stdint.h>
#include <stdarg.h>
#include <stdio.h>

#include "jf_layers.h"

typedef uint16_t bf16_t;

int jl_fail(int code, const char *fmt, ...);       // records the message for jl_last_error(), returns `code`
int jl_check_launch(const char *what);

template <typename T> __device__ __forceinline__ float ld_f(const T *p);
template <> __device__ __forceinline__ float ld_f<float>(const float *p) { return *p; }
template <> __device__ __forceinline__ float ld_f<bf16_t>(const bf16_t *p) { return __uint_as_float(((uint32_t)*p) << 16); }
template <typename T> __device__ __forceinline__ void st_f(T *p, float v);
template <> __device__ __forceinline__ void st_f<float>(float *p, float v) { *p = v; }
template <> __device__ __forceinline__ void st_f<bf16_t>(bf16_t *p, float v) {          // round to nearest even
    uint32_t u = __float_as_uint(v);
    if ((u & 0x7fffffffu) > 0x7f800000u) { *p = 0x7FC0; return; }
    u += 0x7FFFu + ((u >> 16) & 1u);
    *p = (bf16_t)(u >> 16);
}
__device__ __forceinline__ float ld_any(const void *p, int dtype, int64_t i) {
    return dtype == JL_BF16 ? ld_f((const bf16_t *)p + i) : ((const float *)p)[i];
}

// four elements at a time (8 bytes of bfloat16, 16 of float, aligned to that)
__device__ __forceinline__ void ld4_f(const float *p, float (&v)[4]) { const float4 t = *(const float4 *)p; v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w; }
__device__ __forceinline__ void ld4_f(const bf16_t *p, float (&v)[4]) {
    const uint2 t = *(const uint2 *)p;
    v[0] = __uint_as_float(t.x << 16); v[1] = __uint_as_float(t.x & 0xffff0000u); v[2] = __uint_as_float(t.y << 16); v[3] = __uint_as_float(t.y & 0xffff0000u);
}
__device__ __forceinline__ void st4_f(float *p, const float (&v)[4]) { *(float4 *)p = make_float4(v[0], v[1], v[2], v[3]); }
__device__ __forceinline__ void st4_f(bf16_t *p, const float (&v)[4]) {
    bf16_t h[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) st_f(h + i, v[i]);
    *(uint2 *)p = make_uint2((uint32_t)h[0] | ((uint32_t)h[1] << 16), (uint32_t)h[2] | ((uint32_t)h[3] << 16));
}

__device__ __forceinline__ float wave_sum_f32(float v) {
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) v += __shfl_xor(v, off, 64);
    return v;
}
// sum over a workgroup of up to 1024 threads; `red` holds 16 floats of LDS.  Every thread gets the result; the order of
// the additions is fixed by the lane / wavefront numbers.
__device__ __forceinline__ float block_sum_f32(float v, float *red) {
    v = wave_sum_f32(v);
    const int wave = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[wave] = v;
    __syncthreads();
    float s = 0.f;
    for (int i = 0; i < nw; ++i) s += red[i];
    return s;
}

// cap * tanh(s / cap) with tanh(z) = 1 - 2 / (1 + exp(2 z)): a few 1e-7 of cap off, for scores that bfloat16 operands made
__device__ __forceinline__ float soft_cap_fast(float s, float cap) {
    return cap - 2.0f * cap * __builtin_amdgcn_rcpf(1.0f + __expf(2.0f * s * __builtin_amdgcn_rcpf(cap)));
}
// the same for |s| <= cap / 4 without a transcendental: s (1 - z^2/3 + 2 z^4/15 - 17 z^6/315 + 62 z^8/2835), z = s / cap
__device__ __forceinline__ float soft_cap_small(float s, float inv_cap) {
    const float z = s * inv_cap, y = z * z;
    return s * (1.0f + y * (-0.33333333f + y * (0.13333333f + y * (-0.053968254f + y * 0.021869489f))));
}
__device__ __forceinline__ float softplus_f(float z) { return z > 20.f ? z : log1pf(expf(z)); }

// gated units of a feed-forward (jl_gated_act, and the grouped product that applies them in its epilogue)
// FAST: the sigmoid on the hardware's exponential and reciprocal (a few 1e-7 off), for results that are rounded to bfloat16
template <bool FAST = false> __device__ __forceinline__ float sigmoid_f(float z) {
    if (FAST) return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.44269504f * z));
    return 1.0f / (1.0f + expf(-z));
}
// 0.5 z (1 + tanh(u)) = z sigmoid(2u), u = sqrt(2/pi) (z + 0.044715 z^3)
template <bool FAST = false> __device__ __forceinline__ float gelu_tanh_f(float z) {
    return z * sigmoid_f<FAST>(1.5957691216057308f * (z + 0.044715f * z * z * z));
}
__device__ __forceinline__ float gelu_erf_f(float z) { return 0.5f * z * (1.0f + erff(z * 0.70710678118654752f)); }
template <bool FAST = false> __device__ __forceinline__ float silu_f(float z) { return z * sigmoid_f<FAST>(z); }
template <bool FAST = false>
__device__ __forceinline__ float gated_unit_f(float g, float u, int kind, float limit, float alpha, float shift) {
    if (kind == JL_ACT_GELU_TANH) return gelu_tanh_f<FAST>(g) * u;
    if (kind == JL_ACT_SILU) return silu_f<FAST>(g) * u;
    if (kind == JL_ACT_GELU_ERF) return gelu_erf_f(g) * u;
    g = fminf(g, limit);                                            // clamped swish: the gate capped from above, the linear branch from both sides
    u = fminf(fmaxf(u, -limit), limit);
    return g * sigmoid_f<FAST>(alpha * g) * (u + shift);
}

#define JL_DISPATCH(dtype, ...)                                   \
    do {                                                          \
        if ((dtype) == JL_BF16) { typedef bf16_t T; __VA_ARGS__; } \
        else { typedef float T; __VA_ARGS__; }                    \
    } while (0)

#endif
