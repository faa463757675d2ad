// What the delta rules' kernels have in common: pieces of a state column, and the fp32 matrix instruction that sixteen tokens (a
// chunk) go through at a time.
#pragma once
#include "common.h"

namespace {

constexpr float kUnitEps = 1e-6f;  // under the root that makes a key a unit vector
constexpr int kChunk = 16;

typedef float f32x4 __attribute__((ext_vector_type(4)));

struct Vec8 {
    float v[8];
    __device__ __forceinline__ void load(const float* p) {
        const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
        v[0] = a.x, v[1] = a.y, v[2] = a.z, v[3] = a.w, v[4] = b.x, v[5] = b.y, v[6] = b.z, v[7] = b.w;
    }
    __device__ __forceinline__ void store(float* p) const {
        *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
        *reinterpret_cast<float4*>(p + 4) = make_float4(v[4], v[5], v[6], v[7]);
    }
};

template <int L>
__device__ __forceinline__ float dot_over_lanes(const Vec8& a, const Vec8& s) {
    float x = a.v[0] * s.v[0], y = a.v[1] * s.v[1];
#pragma unroll
    for (int j = 2; j < 8; j += 2) x = fmaf(a.v[j], s.v[j], x), y = fmaf(a.v[j + 1], s.v[j + 1], y);
    return lane_group_sum<L>(x + y);
}

__device__ __forceinline__ f32x4 mma(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
__device__ __forceinline__ f32x4 load4(const float* p) { return *reinterpret_cast<const f32x4*>(p); }

}  // namespace
