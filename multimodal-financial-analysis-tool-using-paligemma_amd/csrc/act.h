// act.h -- activation element access shared by the runtime-shape kernels: T is uint16_t (bf16 bits) or float.
#pragma once
#include "common.h"

namespace pgmi {

__device__ __forceinline__ float ldf(const uint16_t* p) { return bf2f(*p); }
__device__ __forceinline__ float ldf(const float* p) { return *p; }
__device__ __forceinline__ void stf(uint16_t* p, float v) { *p = f2bf(v); }
__device__ __forceinline__ void stf(float* p, float v) { *p = v; }

// 8 consecutive elements; p 16-byte aligned (bf16) / 32-byte chunks read as two 16-byte halves (fp32)
__device__ __forceinline__ void ld8(const uint16_t* p, float (&v)[8]) {
    const uint4 u = *reinterpret_cast<const uint4*>(p);
    const uint32_t w[4] = {u.x, u.y, u.z, u.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        v[2 * i] = __uint_as_float(w[i] << 16);
        v[2 * i + 1] = __uint_as_float(w[i] & 0xFFFF0000u);
    }
}
__device__ __forceinline__ void ld8(const float* p, float (&v)[8]) {
    const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
    v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
    v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
}
__device__ __forceinline__ void st8(uint16_t* p, const float (&v)[8]) {
    uint32_t w[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) w[i] = (uint32_t)f2bf(v[2 * i]) | ((uint32_t)f2bf(v[2 * i + 1]) << 16);
    *reinterpret_cast<uint4*>(p) = make_uint4(w[0], w[1], w[2], w[3]);
}
__device__ __forceinline__ void st8(float* p, const float (&v)[8]) {
    *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
    *reinterpret_cast<float4*>(p + 4) = make_float4(v[4], v[5], v[6], v[7]);
}

// 1 / (1 + exp(-x)) with the hardware reciprocal (1 ulp); exp overflowing to +inf gives 0
__device__ __forceinline__ float sigmoidf_(float x) { return __builtin_amdgcn_rcpf(1.0f + __expf(-x)); }
__device__ __forceinline__ float siluf_(float x) { return x * sigmoidf_(x); }
// ln(1 + exp(x)) without overflow or cancellation
__device__ __forceinline__ float softplusf_(float x) { return fmaxf(x, 0.0f) + log1pf(__expf(-fabsf(x))); }
// the same from the hardware exponential and logarithm: a short series where 1 + e would round e away
__device__ __forceinline__ float softplus_fast(float x) {
    const float e = __expf(-fabsf(x));
    const float series = e * (1.0f - e * (0.5f - e * (0.33333333f - e * (0.25f - e * 0.2f))));
    return fmaxf(x, 0.0f) + (e < 0.0625f ? series : __logf(1.0f + e));
}
template <typename T>
__device__ __forceinline__ float softplus_of(float x);
template <>
__device__ __forceinline__ float softplus_of<float>(float x) { return softplusf_(x); }
template <>
__device__ __forceinline__ float softplus_of<uint16_t>(float x) { return softplus_fast(x); }

__device__ __forceinline__ void ld4(const uint16_t* p, float (&v)[4]) {
    const ushort4 u = *reinterpret_cast<const ushort4*>(p);
    v[0] = bf2f(u.x); v[1] = bf2f(u.y); v[2] = bf2f(u.z); v[3] = bf2f(u.w);
}
__device__ __forceinline__ void ld4(const float* p, float (&v)[4]) {
    const float4 u = *reinterpret_cast<const float4*>(p);
    v[0] = u.x; v[1] = u.y; v[2] = u.z; v[3] = u.w;
}
__device__ __forceinline__ void st4(uint16_t* p, const float (&v)[4]) {
    *reinterpret_cast<ushort4*>(p) = make_ushort4(f2bf(v[0]), f2bf(v[1]), f2bf(v[2]), f2bf(v[3]));
}
__device__ __forceinline__ void st4(float* p, const float (&v)[4]) {
    *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
}

// minGRU's candidate: u + 1/2 for u >= 0, sigmoid(u) below
__device__ __forceinline__ float gru_candidate(float u) { return u >= 0.0f ? u + 0.5f : sigmoidf_(u); }

}  // namespace pgmi
