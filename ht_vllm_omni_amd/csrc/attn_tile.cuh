// What the transposed-operand attention kernels share (latent_attn.hip, window_attn.hip): lane (c = lane & 15, qk = lane >> 4) owns query row c from the
// scores to the store; the softmax weights are fp32 and enter the second product as three bf16 terms whose sum is the fp32 value.
#pragma once
#include "common.cuh"
#include "gemm_frag.cuh"

#define LA_KEYS 32
#define LA_LOG2E 1.4426950408889634f
#define LA_DEC_WAVES 4
#define LA_MAX_SPLIT 16
#define LA_SENT (-1e30f)

typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) s16x4 lds_s16x4;

// KV splits a row of `ntiles` 16-key tiles uses, of the nsplit the launch offers: two rounds of the four waves each, or more
__device__ __forceinline__ int la_row_splits(int ntiles, int nsplit) { return min(nsplit, (ntiles + 7) / 8); }

// a pair of fp32 values as three bf16 terms each
__device__ __forceinline__ void split3(float a, float b, uint32_t& hi, uint32_t& mid, uint32_t& lo) {
    hi = pack_bf2(a, b);
    const float ar = a - bf_lo(hi), br = b - bf_hi(hi);
    mid = pack_bf2(ar, br);
    lo = pack_bf2(ar - bf_lo(mid), br - bf_hi(mid));
}

// 2^x of weights and decays (one instruction; below 2^-126: zero)
__device__ __forceinline__ float exp2_w(float x) { return __builtin_amdgcn_exp2f(x); }

// key of contraction slot (qk, j) inside a 32-key tile
__device__ __forceinline__ int la_slot(int qk, int j) { return j < 4 ? 4 * qk + j : 16 + 4 * qk + (j - 4); }

// transposed fragment out of a row-major bf16 tile (rows = contraction slots, `pitch` bytes apart): lane (c, qk) gets column 16 ct + c of its 8 rows
__device__ __forceinline__ u32x4 la_transposed_at(const unsigned char* img, int pitch, int ct, int c, int qk) {
    const unsigned char* p = img + (4 * qk + (c >> 2)) * pitch + (16 * ct + (c & 3) * 4) * 2;
    const s16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)p);
    const s16x4 b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)(p + 16 * pitch));
    const u32x2 x = __builtin_bit_cast(u32x2, a), y = __builtin_bit_cast(u32x2, b);
    return (u32x4){x[0], x[1], y[0], y[1]};
}

// workgroups of a decode launch -> KV splits: two workgroups per CU, at least one 16-key tile per wave and split
static inline int la_split_count(int wgs, int max_keys) {
    int ns = 512 / (wgs > 0 ? wgs : 1);
    const int cap = (max_keys + 63) / 64;
    if (ns > cap) ns = cap;
    if (ns > LA_MAX_SPLIT) ns = LA_MAX_SPLIT;
    return ns < 1 ? 1 : ns;
}
