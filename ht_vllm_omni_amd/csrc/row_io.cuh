// Four consecutive values of a row, whatever it is made of: bf16 or fp32 elements, or the partial sums of a product (decoder_rows.hip, decay_rec.hip).
#pragma once
#include "common.cuh"
#include "../../include/omni_decoder.h"

// ---- element type of matrix operands: 4 consecutive values
template <typename E>
__device__ __forceinline__ void ld4(const E* p, float (&v)[4]);
template <>
__device__ __forceinline__ void ld4<float>(const float* p, float (&v)[4]) {
    const float4 a = *reinterpret_cast<const float4*>(p);
    v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
}
template <>
__device__ __forceinline__ void ld4<uint16_t>(const uint16_t* p, float (&v)[4]) {
    const uint2 a = *reinterpret_cast<const uint2*>(p);
    v[0] = bf_lo(a.x); v[1] = bf_hi(a.x); v[2] = bf_lo(a.y); v[3] = bf_hi(a.y);
}
template <typename E>
__device__ __forceinline__ void st4(E* p, const float (&v)[4]);
template <>
__device__ __forceinline__ void st4<float>(float* p, const float (&v)[4]) { *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]); }
template <>
__device__ __forceinline__ void st4<uint16_t>(uint16_t* p, const float (&v)[4]) {
    *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3]));
}

// 4 consecutive values of an array that arrives as `slabs` partial sums `stride` elements apart, added in slab order.  More than one: all
// OMNI_STREAM_MAX_SPLITS loads leave at once (past the last slab: a repeated address, not added)
__device__ __forceinline__ void ld4_slabs(const float* p, int slabs, int64_t stride, float (&v)[4]) {
    ld4<float>(p, v);
    if (slabs <= 1) return;
    float z[OMNI_STREAM_MAX_SPLITS][4];
#pragma unroll
    for (int s = 1; s < OMNI_STREAM_MAX_SPLITS; ++s) ld4<float>(p + min(s, slabs - 1) * stride, z[s]);
#pragma unroll
    for (int s = 1; s < OMNI_STREAM_MAX_SPLITS; ++s)
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] += s < slabs ? z[s][e] : 0.f;
}
