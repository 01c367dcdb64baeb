// Shared helpers of the gfx950 kernel library: dtype codes, error reporting, bf16 <-> f32,
// wave and block reductions.  Wavefronts are 64 lanes wide.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>
#include <stdio.h>
#include <stdarg.h>
#include <math.h>

#define SPY_F32 0
#define SPY_BF16 1
#define SPY_WAVE 64

typedef uint16_t bf16_t;

extern "C" const char* spy_last_error();
int spy_fail(const char* fmt, ...);   // records the message, returns 1

#define SPY_REQUIRE(cond, ...)              \
    do {                                    \
        if (!(cond)) return spy_fail(__VA_ARGS__); \
    } while (0)

#define SPY_CHECK_LAUNCH(name)                                                        \
    do {                                                                              \
        hipError_t e_ = hipGetLastError();                                            \
        if (e_ != hipSuccess) return spy_fail("%s: launch failed: %s", name, hipGetErrorString(e_)); \
    } while (0)

__device__ __forceinline__ float bf16_to_f32(bf16_t x) { return __uint_as_float(((uint32_t)x) << 16); }

// round to nearest, ties to even; NaN stays NaN.  gfx950 converts in hardware (v_cvt_pk_bf16_f32).
__device__ __forceinline__ bf16_t f32_to_bf16(float f) { return __builtin_bit_cast(unsigned short, (__bf16)f); }

// two values in one instruction: a in the low half, b in the high half
__device__ __forceinline__ uint32_t pack_bf16x2(float a, float b) {
    typedef float f32x2_ __attribute__((ext_vector_type(2)));
    typedef __bf16 bf16x2_ __attribute__((ext_vector_type(2)));
    const f32x2_ v = {a, b};
    return __builtin_bit_cast(uint32_t, __builtin_convertvector(v, bf16x2_));
}

template <typename T> __device__ __forceinline__ float to_f32(T x);
template <> __device__ __forceinline__ float to_f32<float>(float x) { return x; }
template <> __device__ __forceinline__ float to_f32<bf16_t>(bf16_t x) { return bf16_to_f32(x); }

template <typename T> __device__ __forceinline__ T from_f32(float x);
template <> __device__ __forceinline__ float from_f32<float>(float x) { return x; }
template <> __device__ __forceinline__ bf16_t from_f32<bf16_t>(float x) { return f32_to_bf16(x); }

// four consecutive values as floats, moved as one 16-byte (float32) or 8-byte (bfloat16) piece; the address is aligned so
template <typename TA> struct Vec4;
template <> struct Vec4<float> {
    typedef float4 type;
    static __device__ __forceinline__ void load(const float* p, float* v) { const float4 t = *reinterpret_cast<const float4*>(p); v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w; }
    static __device__ __forceinline__ void store(float* p, const float* v) { *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]); }
};
template <> struct Vec4<bf16_t> {
    static __device__ __forceinline__ void load(const bf16_t* p, float* v) {
        const uint2 t = *reinterpret_cast<const uint2*>(p);
        v[0] = __uint_as_float(t.x << 16); v[1] = __uint_as_float(t.x & 0xffff0000u);
        v[2] = __uint_as_float(t.y << 16); v[3] = __uint_as_float(t.y & 0xffff0000u);
    }
    static __device__ __forceinline__ void store(bf16_t* p, const float* v) {
        uint2 t;
        t.x = (uint32_t)f32_to_bf16(v[0]) | ((uint32_t)f32_to_bf16(v[1]) << 16);
        t.y = (uint32_t)f32_to_bf16(v[2]) | ((uint32_t)f32_to_bf16(v[3]) << 16);
        *reinterpret_cast<uint2*>(p) = t;
    }
};

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

// Block-wide sum; `red` is shared memory of at least blockDim.x / 64 floats.  Every thread gets the result.
__device__ __forceinline__ float block_sum(float v, float* red) {
    v = wave_sum(v);
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
    __syncthreads();
    if (lane == 0) red[w] = v;
    __syncthreads();
    float t = 0.f;
    for (int i = 0; i < nw; ++i) t += red[i];
    return t;
}
__device__ __forceinline__ float block_max(float v, float* red) {
    v = wave_max(v);
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
    __syncthreads();
    if (lane == 0) red[w] = v;
    __syncthreads();
    float t = red[0];
    for (int i = 1; i < nw; ++i) t = fmaxf(t, red[i]);
    return t;
}

// xIELU with the numbers ap = softplus(p), aq = 1/2 + softplus(q):  z > 0: ap z^2 + z/2;  z <= 0: aq (e^z - 1 - z) + z/2
__device__ __forceinline__ float softplus_f(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
__device__ __forceinline__ float xielu_f(float z, float ap, float aq) {
    return z > 0.f ? fmaf(ap * z, z, 0.5f * z) : fmaf(aq, expm1f(z) - z, 0.5f * z);
}

__device__ __forceinline__ float gelu_f(float z) { return 0.5f * z * (1.0f + erff(z * 0.7071067811865476f)); }

// The activation of a gated feed-forward, z sigmoid(z (c1 + c3 z^2)) of the gate's value z:  silu with (1, 0), and the tanh
// form of gelu, z/2 (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3))), with twice the tanh's two factors, 1 + tanh(y) being
// 2 sigmoid(2 y).  The kernels take the two numbers and have no branch.
struct GateAct { float c1, c3; };
#define SPY_ACT_SILU 0
#define SPY_ACT_GELU_TANH 1
#define SPY_ACT_GELU 2           // the exact gelu, z/2 (1 + erf(z / sqrt 2)): products without a gate only
inline bool gate_act_of(int code, GateAct* a) {
    if (code == SPY_ACT_SILU) { *a = {1.0f, 0.0f}; return true; }
    if (code == SPY_ACT_GELU_TANH) { *a = {1.5957691216057308f, 0.07135481282553525f}; return true; }
    return false;
}
__device__ __forceinline__ float gated_value(const GateAct& a, float z, float up) {
    return (z / (1.0f + expf(-(z * fmaf(a.c3 * z, z, a.c1))))) * up;
}

// Dispatch on a dtype code: binds `T` in `body`.
#define SPY_DISPATCH(code, T, ...)                  \
    if ((code) == SPY_F32) { typedef float T; __VA_ARGS__; } \
    else { typedef bf16_t T; __VA_ARGS__; }
