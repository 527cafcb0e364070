// Shared helpers of the gfx950 kernels: element types, conversions, wave reductions and the error
// channel of the C entry points.  Every entry point returns 0 on success and -1 after storing a
// message that ilm_last_error() returns.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>
#include <stdio.h>

#define ILM_DTYPE_F32 0
#define ILM_DTYPE_BF16 1

#define WAVE 64

struct bf16 {
    uint16_t bits;
};

__device__ __host__ __forceinline__ float bf16_bits_to_f32(uint16_t b) {
    union {
        uint32_t u;
        float f;
    } c;
    c.u = ((uint32_t)b) << 16;
    return c.f;
}

// round to nearest even; NaN stays NaN
__device__ __host__ __forceinline__ uint16_t f32_to_bf16_bits(float f) {
    union {
        uint32_t u;
        float f;
    } c;
    c.f = f;
    uint32_t u = c.u;
    if ((u & 0x7fffffffu) > 0x7f800000u) return (uint16_t)((u >> 16) | 0x40u);
    u += 0x7fffu + ((u >> 16) & 1u);
    return (uint16_t)(u >> 16);
}

__device__ __forceinline__ float to_f32(float v) { return v; }
__device__ __forceinline__ float to_f32(bf16 v) { return bf16_bits_to_f32(v.bits); }

template <typename T>
__device__ __forceinline__ T from_f32(float v);
template <>
__device__ __forceinline__ float from_f32<float>(float v) {
    return v;
}
template <>
__device__ __forceinline__ bf16 from_f32<bf16>(float v) {
    // the hardware's conversion (round to nearest even), one instruction on gfx950
    bf16 r;
    r.bits = __builtin_bit_cast(uint16_t, (__bf16)v);
    return r;
}

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
    return v;
}
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, 64));
    return v;
}

// Sum over a block of NW waves; every thread gets the result.  `red` holds NW floats of LDS.
template <int NW>
__device__ __forceinline__ float block_sum(float v, float* red) {
    v = wave_sum(v);
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
    __syncthreads();
    if (lane == 0) red[w] = v;
    __syncthreads();
    float t = 0.f;
#pragma unroll
    for (int i = 0; i < NW; ++i) t += red[i];
    return t;
}

// The first key a token at position p sees.  `reach` > 0: its last `reach` positions; < 0: the positions of its own chunk, chunks
// of -reach positions counted from the sequence's start; 0: all.  It never falls as p grows.
__device__ __forceinline__ int first_key(int p, int reach) {
    if (reach > 0) return p - reach + 1 > 0 ? p - reach + 1 : 0;
    return reach < 0 ? p - p % -reach : 0;
}

// Activations
__device__ __forceinline__ float silu_f(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float sigmoid_f(float x) { return 1.0f / (1.0f + expf(-x)); }

#define ILM_ACT_NONE 0
#define ILM_ACT_SILU 1
#define ILM_ACT_SIGMOID 2
#define ILM_ACT_RELU2 3
#define ILM_ACT_GELU_TANH 4

__device__ __forceinline__ float act_f(float x, int kind) {
    switch (kind) {
        case ILM_ACT_SILU: return silu_f(x);
        case ILM_ACT_SIGMOID: return sigmoid_f(x);
        case ILM_ACT_RELU2: { const float r = fmaxf(x, 0.f); return r * r; }
        case ILM_ACT_GELU_TANH: return 0.5f * x * (1.0f + tanhf(0.7978845608028654f * (x + 0.044715f * x * x * x)));
        default: return x;
    }
}

// The gate's activation of a gated feed-forward
#define ILM_GLU_SILU 0
#define ILM_GLU_GELU_TANH 1
// (both are g * sigmoid(z): z = g, or twice the argument of the tanh)
__device__ __forceinline__ float glu_act(float g, int kind) {
    const float z = kind == ILM_GLU_GELU_TANH ? 1.5957691216057308f * (g + 0.044715f * g * g * g) : g;
    return g / (1.0f + expf(-z));
}

extern "C" const char* ilm_last_error();
void ilm_set_error(const char* fmt, ...);
// compute units of the current device (looked up once a process; 256 if the runtime does not say)
int ilm_num_cus();

#define ILM_REQUIRE(cond, ...)          \
    do {                                \
        if (!(cond)) {                  \
            ilm_set_error(__VA_ARGS__); \
            return -1;                  \
        }                               \
    } while (0)

#define ILM_LAUNCH_CHECK(name)                                                   \
    do {                                                                         \
        hipError_t e__ = hipGetLastError();                                      \
        if (e__ != hipSuccess) {                                                 \
            ilm_set_error("%s: launch failed: %s", name, hipGetErrorString(e__)); \
            return -1;                                                           \
        }                                                                        \
    } while (0)
