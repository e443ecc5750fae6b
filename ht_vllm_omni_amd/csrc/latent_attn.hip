// Causal attention over a paged cache of latents shared by all heads (include/omni_decoder.h omni_latent_attn): the keys ARE the values, so
// a cache row is read once for both products, and every (token, head) pair of a sequence is one query row of the same matrix problem.
//
// Matrix-core form (bf16 cache, rp = 32 * RS): v_mfma_f32_16x16x32_bf16, both products TRANSPOSED so that a lane owns one query row from the
// first MFMA to the store:
//   S^T[key][row] = C . Q^T      A = C (lane (key, chunk qk): 8 dims, ds_read_b128), B = Q^T (registers for the whole kernel)
//   O^T[d][row]  += C^T . P^T    B = P^T: the contraction slot (qk, j) is DEFINED as key (j < 4 ? 4 qk + j : 16 + 4 qk + j - 4) -- the
//                                scores the lane already holds; A = C^T: the same keys at one d, ds_read_b64_tr_b16 out of the
//                                row-major tile (a 16-lane group reads 4 rows x 32 B and gets them transposed)
// Scores, softmax statistics and weights are fp32; the weights enter the second product as three bf16 terms whose sum is the fp32 value.
//
//   latent_decode_kernel   one token: up to 16 heads fill the 16 query rows; every wave walks its own 32-key tiles (private LDS image, no
//                          barrier in the loop, the next tile travels in registers), waves and KV splits merge at the end
//   latent_prefill_kernel  tiles of up to 128 query rows of one sequence; PW waves share each 32-key tile (double-buffered, one barrier per
//                          tile), MT 16-row groups per wave
//   latent_plain_kernel    any width, bf16 or fp32: one wave per query row on the vector units (the 32-bit mode)
#include "common.cuh"
#include "gemm_frag.cuh"
#include "../../include/omni_decoder.h"

#define LA_KEYS 32
#define LA_LOG2E 1.4426950408889634f
#define LA_DEC_WAVES 4
#define LA_MAX_SPLIT 16
#define LA_SENT (-1e30f)

typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) s16x4 lds_s16x4;

struct LatentArgs {
    const uint16_t* q; const uint16_t* cache; const float* gate; uint16_t* out;
    const int32_t* block_table; int bt_stride, bs_shift, bs_mask;
    const int32_t* row_of_tok; const int32_t* positions; const int32_t* tiles;
    int heads; float qs;            // scale * log2(e)
    float* partial; int nsplit;
};

template <int RS>
struct LatentGeom {
    static constexpr int ROWB = RS * 64;              // bytes of a cache row
    static constexpr int PITCH = ROWB + 32;           // LDS row pitch: 8 consecutive rows' 32-byte pieces cover all 64 banks
    static constexpr int CH = RS * 4;                 // 16-byte chunks per row
    static constexpr int TILE = LA_KEYS * PITCH;
};

// scores of one 16-row group against the 32-key tile at `img` -> online softmax update -> weights as three bf16 terms
template <int RS>
__device__ __forceinline__ void la_scores(const unsigned char* img, const u32x4 (&Q)[RS], int c, int qk, f32x4 (&S)[2]) {
    constexpr int PITCH = LatentGeom<RS>::PITCH;
#pragma unroll
    for (int kt = 0; kt < 2; ++kt) {
        S[kt] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < RS; ++s) {
            const u32x4 A = *reinterpret_cast<const u32x4*>(img + (16 * kt + c) * PITCH + (32 * s + 8 * qk) * 2);
            S[kt] = mfma16(A, Q[s], S[kt]);
        }
    }
}

struct LaWeights { u32x4 hi, mid, lo; };
// nlive: keys of the tile this row sees (<= 0: none)
__device__ __forceinline__ LaWeights la_softmax(const f32x4 (&S)[2], float qs, int nlive, int qk, float& m, float& l, float& alpha) {
    float sv[8], mx = LA_SENT;
    bool ok[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) {
        const int kidx = (j < 4) ? 4 * qk + j : 16 + 4 * qk + (j - 4);
        sv[j] = S[j >> 2][j & 3] * qs;
        ok[j] = kidx < nlive;
        if (ok[j]) mx = fmaxf(mx, sv[j]);
    }
    mx = xor32_max(xor16_max(mx));
    const float mn = fmaxf(m, mx);
    alpha = exp2f(m - mn);                   // both the sentinel: 1, harmless (l = 0, O = 0)
    float p[8], rs = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
        p[j] = ok[j] ? exp2f(sv[j] - mn) : 0.f;
        rs += p[j];
    }
    rs = xor32_sum(xor16_sum(rs));
    l = l * alpha + rs;
    m = mn;
    LaWeights w;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        const float a = p[2 * e], b = p[2 * e + 1];
        const float ar = a - bfround(a), br = b - bfround(b);
        const float am = bfround(ar), bm = bfround(br);
        w.hi[e] = pack_bf2(a, b);
        w.mid[e] = pack_bf2(am, bm);
        w.lo[e] = pack_bf2(ar - am, br - bm);
    }
    return w;
}

// C^T fragment of d tile dt: lane (d = c, qk) gets the 8 keys of its contraction slots
template <int RS>
__device__ __forceinline__ u32x4 la_transposed(const unsigned char* img, int dt, int c, int qk) {
    constexpr int PITCH = LatentGeom<RS>::PITCH;
    const unsigned char* p = img + (4 * qk + (c >> 2)) * PITCH + (16 * dt + (c & 3) * 4) * 2;
    const s16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)p);
    const s16x4 b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)(p + 16 * PITCH));
    const u32x2 x = __builtin_bit_cast(u32x2, a), y = __builtin_bit_cast(u32x2, b);
    return (u32x4){x[0], x[1], y[0], y[1]};
}

template <int RS>
__global__ __launch_bounds__(64 * LA_DEC_WAVES, 1) void latent_decode_kernel(const LatentArgs a) {
    using G = LatentGeom<RS>;
    constexpr int LOADS = LA_KEYS * G::CH / 64;       // 16-byte loads per lane and tile
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];
    __shared__ float sm[LA_DEC_WAVES][16], sl[LA_DEC_WAVES][16];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int c = lane & 15, qk = lane >> 4;
    const int t = blockIdx.y, split = blockIdx.z;
    const int head = blockIdx.x * 16 + c, hc = min(head, a.heads - 1);
    const int rp = RS * 32;
    unsigned char* img = lds + wave * G::TILE;
    u32x4 Q[RS];
#pragma unroll
    for (int s = 0; s < RS; ++s) Q[s] = ld16(a.q + ((size_t)t * a.heads + hc) * rp + 32 * s + 8 * qk);
    const int len = a.positions[t] + 1;
    const int32_t* bt = a.block_table + (size_t)a.row_of_tok[t] * a.bt_stride;
    const int ntiles = (len + LA_KEYS - 1) / LA_KEYS, step = a.nsplit * LA_DEC_WAVES;
    f32x4 O[2 * RS];
#pragma unroll
    for (int d = 0; d < 2 * RS; ++d) O[d] = (f32x4){0.f, 0.f, 0.f, 0.f};
    float m = LA_SENT, l = 0.f;
    u32x4 st[LOADS];
    auto fetch = [&](int tile) {
        const int key = min(tile * LA_KEYS + (lane & 31), len - 1);          // tail keys: a valid row, masked below
        const int slot = (bt[key >> a.bs_shift] << a.bs_shift) + (key & a.bs_mask);
#pragma unroll
        for (int j = 0; j < LOADS; ++j) {
            const int i = lane + 64 * j;
            const int kk = i / G::CH, ch = i - kk * G::CH;
            const int row = G::CH % 64 == 0 ? __builtin_amdgcn_readlane(slot, j / (G::CH / 64 > 0 ? G::CH / 64 : 1)) : __shfl(slot, kk, 64);
            st[j] = ld16(a.cache + (size_t)row * rp + ch * 8);
        }
    };
    int tile = split * LA_DEC_WAVES + wave;
    if (tile < ntiles) fetch(tile);
    for (; tile < ntiles; tile += step) {
#pragma unroll
        for (int j = 0; j < LOADS; ++j) {
            const int i = lane + 64 * j;
            const int kk = i / G::CH, ch = i - kk * G::CH;
            *reinterpret_cast<u32x4*>(img + kk * G::PITCH + ch * 16) = st[j];
        }
        if (tile + step < ntiles) fetch(tile + step);
        __builtin_amdgcn_wave_barrier();
        f32x4 S[2];
        la_scores<RS>(img, Q, c, qk, S);
        float alpha;
        const LaWeights w = la_softmax(S, a.qs, len - tile * LA_KEYS, qk, m, l, alpha);
        if (__any(alpha != 1.0f)) {
#pragma unroll
            for (int d = 0; d < 2 * RS; ++d) O[d] *= alpha;
        }
#pragma unroll
        for (int d = 0; d < 2 * RS; ++d) {
            const u32x4 VT = la_transposed<RS>(img, d, c, qk);
            O[d] = mfma16(VT, w.hi, mfma16(VT, w.mid, mfma16(VT, w.lo, O[d])));
        }
        __builtin_amdgcn_wave_barrier();
    }
    // ---- the four waves' partial results
    if (qk == 0) { sm[wave][c] = m; sl[wave][c] = l; }
    __syncthreads();                                   // (also: every wave is done with its tile image)
    float M = LA_SENT, L = 0.f;
#pragma unroll
    for (int w = 0; w < LA_DEC_WAVES; ++w) M = fmaxf(M, sm[w][c]);
#pragma unroll
    for (int w = 0; w < LA_DEC_WAVES; ++w) L += sl[w][c] * exp2f(sm[w][c] - M);
    const float f = exp2f(m - M);
    f32x4* ex = reinterpret_cast<f32x4*>(lds);         // [wave][d tile][lane]
#pragma unroll
    for (int d = 0; d < 2 * RS; ++d) ex[(wave * 2 * RS + d) * 64 + lane] = O[d] * f;
    __syncthreads();
    if (head >= a.heads) return;
    const size_t rh = (size_t)t * a.heads + head;
    float* rec = a.nsplit > 1 ? a.partial + (rh * a.nsplit + split) * (rp + 4) : nullptr;
    if (rec && wave == 0 && qk == 0) { rec[0] = M; rec[1] = L; }
    const float inv = (L > 0.f ? 1.0f / L : 0.f) * (a.gate ? a.gate[rh] : 1.0f);
    for (int d = wave; d < 2 * RS; d += LA_DEC_WAVES) {
        f32x4 v = ex[d * 64 + lane];
#pragma unroll
        for (int w = 1; w < LA_DEC_WAVES; ++w) v += ex[(w * 2 * RS + d) * 64 + lane];
        if (rec) {
            *reinterpret_cast<f32x4*>(rec + 4 + 16 * d + 4 * qk) = v;
        } else {
            v *= inv;
            *reinterpret_cast<uint2*>(a.out + rh * rp + 16 * d + 4 * qk) = make_uint2(pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3]));
        }
    }
}

// KV splits of one (token, head)
__global__ __launch_bounds__(64) void latent_merge_kernel(const float* __restrict__ partial, const float* __restrict__ gate, uint16_t* __restrict__ out,
                                                          int nsplit, int rp) {
    const size_t rh = blockIdx.x;
    const float* base = partial + rh * nsplit * (rp + 4);
    float M = LA_SENT, L = 0.f;
    for (int s = 0; s < nsplit; ++s) M = fmaxf(M, base[(size_t)s * (rp + 4)]);
    for (int s = 0; s < nsplit; ++s) L += base[(size_t)s * (rp + 4) + 1] * exp2f(base[(size_t)s * (rp + 4)] - M);
    const float inv = (L > 0.f ? 1.0f / L : 0.f) * (gate ? gate[rh] : 1.0f);
    for (int k = threadIdx.x * 4; k < rp; k += 256) {
        f32x4 v = (f32x4){0.f, 0.f, 0.f, 0.f};
        for (int s = 0; s < nsplit; ++s) {
            const float* rec = base + (size_t)s * (rp + 4);
            v += *reinterpret_cast<const f32x4*>(rec + 4 + k) * exp2f(rec[0] - M);
        }
        v *= inv;
        *reinterpret_cast<uint2*>(out + rh * rp + k) = make_uint2(pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3]));
    }
}

template <int RS, int PW, int MT>
__global__ __launch_bounds__(64 * PW, PW / 4) void latent_prefill_kernel(const LatentArgs a) {
    using G = LatentGeom<RS>;
    static_assert(PW * MT * 16 == OMNI_LATENT_TILE, "a work item is one tile of query rows");
    constexpr int NT = 64 * PW, ITEMS = LA_KEYS * G::CH, LOADS = (ITEMS + NT - 1) / NT;
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];      // two tile images
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int c = lane & 15, qk = lane >> 4;
    const int row0 = a.tiles[2 * blockIdx.x], nrows = a.tiles[2 * blockIdx.x + 1];
    const int rp = RS * 32;
    const int32_t* bt = a.block_table + (size_t)a.row_of_tok[row0 / a.heads] * a.bt_stride;
    u32x4 Q[MT][RS];
    f32x4 O[MT][2 * RS];
    float m[MT], l[MT];
    int see[MT], wsee = 0;                              // keys a row sees; most keys any row of this wave sees
    size_t frow[MT];
#pragma unroll
    for (int i = 0; i < MT; ++i) {
        const int r = (wave * MT + i) * 16 + c;
        frow[i] = (size_t)(row0 + min(r, nrows - 1));
        see[i] = r < nrows ? a.positions[frow[i] / a.heads] + 1 : 0;
        m[i] = LA_SENT;
        l[i] = 0.f;
#pragma unroll
        for (int s = 0; s < RS; ++s) Q[i][s] = ld16(a.q + frow[i] * rp + 32 * s + 8 * qk);
#pragma unroll
        for (int d = 0; d < 2 * RS; ++d) O[i][d] = (f32x4){0.f, 0.f, 0.f, 0.f};
        const int last = min((wave * MT + i) * 16 + 15, nrows - 1);
        if ((wave * MT + i) * 16 < nrows) wsee = max(wsee, a.positions[(row0 + last) / a.heads] + 1);
    }
    const int nkeys = a.positions[(row0 + nrows - 1) / a.heads] + 1;
    u32x4 st[LOADS];
    auto fetch = [&](int k0) {
#pragma unroll
        for (int j = 0; j < LOADS; ++j) {
            const int i = threadIdx.x + NT * j;
            if (ITEMS % NT != 0 && i >= ITEMS) continue;
            const int kk = i / G::CH, ch = i - kk * G::CH;
            const int key = min(k0 + kk, nkeys - 1);
            const size_t row = ((size_t)bt[key >> a.bs_shift] << a.bs_shift) + (key & a.bs_mask);
            st[j] = ld16(a.cache + row * rp + ch * 8);
        }
    };
    fetch(0);
    int buf = 0;
    for (int k0 = 0; k0 < nkeys; k0 += LA_KEYS, buf ^= 1) {
        unsigned char* img = lds + buf * G::TILE;
#pragma unroll
        for (int j = 0; j < LOADS; ++j) {
            const int i = threadIdx.x + NT * j;
            if (ITEMS % NT != 0 && i >= ITEMS) continue;
            const int kk = i / G::CH, ch = i - kk * G::CH;
            *reinterpret_cast<u32x4*>(img + kk * G::PITCH + ch * 16) = st[j];
        }
        if (k0 + LA_KEYS < nkeys) fetch(k0 + LA_KEYS);
        __syncthreads();                                // image `buf` complete; image `buf ^ 1` is rewritten only behind the NEXT barrier's arrivals
        if (k0 >= wsee) continue;                       // (wave-uniform; the barriers above stay common)
        LaWeights w[MT];
#pragma unroll
        for (int i = 0; i < MT; ++i) {
            f32x4 S[2];
            la_scores<RS>(img, Q[i], c, qk, S);
            float alpha;
            w[i] = la_softmax(S, a.qs, see[i] - k0, qk, m[i], l[i], alpha);
            if (__any(alpha != 1.0f)) {
#pragma unroll
                for (int d = 0; d < 2 * RS; ++d) O[i][d] *= alpha;
            }
        }
#pragma unroll
        for (int d = 0; d < 2 * RS; ++d) {
            const u32x4 VT = la_transposed<RS>(img, d, c, qk);
#pragma unroll
            for (int i = 0; i < MT; ++i) O[i][d] = mfma16(VT, w[i].hi, mfma16(VT, w[i].mid, mfma16(VT, w[i].lo, O[i][d])));
        }
    }
#pragma unroll
    for (int i = 0; i < MT; ++i) {
        if (see[i] <= 0) continue;
        const float inv = 1.0f / l[i] * (a.gate ? a.gate[frow[i]] : 1.0f);
#pragma unroll
        for (int d = 0; d < 2 * RS; ++d) {
            const f32x4 v = O[i][d] * inv;
            *reinterpret_cast<uint2*>(a.out + frow[i] * rp + 16 * d + 4 * qk) = make_uint2(pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3]));
        }
    }
}

// ---- any width, bf16 or fp32 elements: one wave per (token, head), 64 keys per pass (lane = key for the scores, lane = dims for the sum)
template <typename E>
__device__ __forceinline__ float la_ld(const E* p, size_t i);
template <>
__device__ __forceinline__ float la_ld<float>(const float* p, size_t i) { return p[i]; }
template <>
__device__ __forceinline__ float la_ld<uint16_t>(const uint16_t* p, size_t i) { return bf2f(p[i]); }

#define LA_PLAIN_MAX 1024
template <typename E>
__global__ __launch_bounds__(64) void latent_plain_kernel(const E* __restrict__ q, const E* __restrict__ cache, const float* __restrict__ gate, E* __restrict__ out,
                                                          const int32_t* __restrict__ block_table, int bt_stride, int bs, const int32_t* __restrict__ row_of_tok,
                                                          const int32_t* __restrict__ positions, int heads, int rp, float scale) {
    __shared__ float sq[LA_PLAIN_MAX], sp[64];
    __shared__ int srow[64];
    constexpr int NI = LA_PLAIN_MAX / 64;
    const int lane = threadIdx.x;
    const size_t rh = blockIdx.x;
    const int t = (int)(rh / heads);
    for (int k = lane; k < rp; k += 64) sq[k] = la_ld(q, rh * rp + k);
    const int len = positions[t] + 1;
    const int32_t* bt = block_table + (size_t)row_of_tok[t] * bt_stride;
    float m = LA_SENT, l = 0.f, acc[NI];
#pragma unroll
    for (int i = 0; i < NI; ++i) acc[i] = 0.f;
    for (int k0 = 0; k0 < len; k0 += 64) {
        __syncthreads();                               // one wave per workgroup: orders the LDS traffic of the passes
        const int key = k0 + lane, kc = min(key, len - 1);
        const int row = bt[kc / bs] * bs + kc % bs;
        float s = 0.f;
        for (int k = 0; k < rp; ++k) s = fmaf(sq[k], la_ld(cache, (size_t)row * rp + k), s);
        s *= scale;
        const bool ok = key < len;
        const float mn = fmaxf(m, wave_max(ok ? s : LA_SENT));
        const float alpha = expf(m - mn), p = ok ? expf(s - mn) : 0.f;
        l = l * alpha + wave_sum(p);
        m = mn;
        sp[lane] = p;
        srow[lane] = row;
        __syncthreads();
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            const int d = lane + 64 * i;
            if (d >= rp) continue;
            float v = acc[i] * alpha;
            for (int u = 0; u < 64; ++u) v = fmaf(sp[u], la_ld(cache, (size_t)srow[u] * rp + d), v);
            acc[i] = v;
        }
    }
    const float inv = 1.0f / l * (gate ? gate[rh] : 1.0f);
#pragma unroll
    for (int i = 0; i < NI; ++i) {
        const int d = lane + 64 * i;
        if (d >= rp) continue;
        if constexpr (sizeof(E) == 4) out[rh * rp + d] = acc[i] * inv;
        else out[rh * rp + d] = f2bf(acc[i] * inv);
    }
}

// ---- host side
static int la_splits(int n_decode, int heads, int max_keys) {
    const int wgs = n_decode * ((heads + 15) / 16);
    int ns = 256 / (wgs > 0 ? wgs : 1);
    const int cap = (max_keys + 127) / 128;             // at least one tile per wave and split
    if (ns > cap) ns = cap;
    if (ns > LA_MAX_SPLIT) ns = LA_MAX_SPLIT;
    return ns < 1 ? 1 : ns;
}

extern "C" int64_t omni_latent_attn_workspace_bytes(int n_decode, int heads, int rp) {
    return (int64_t)n_decode * heads * LA_MAX_SPLIT * (rp + 4) * (int64_t)sizeof(float);
}

#define LA_WIDTHS(X) X(1) X(2) X(3) X(4) X(5) X(6) X(7) X(8) X(10) X(12) X(14) X(16)
extern "C" int omni_latent_attn_mfma(int rp) {
#define X(RS_) if (rp == RS_ * 32) return 1;
    LA_WIDTHS(X)
#undef X
    return 0;
}

template <typename K>
static int la_lds(K kernel, int bytes) {
    if (bytes <= 64 * 1024) return OMNI_OK;
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, bytes);
    if (e != hipSuccess) { omni_set_error("omni_latent_attn: LDS attribute: %s", hipGetErrorString(e)); return OMNI_EHIP; }
    return OMNI_OK;
}

template <int RS>
static int la_run(const omni_latent_attn& p, LatentArgs a, hipStream_t st) {
    using G = LatentGeom<RS>;
    if (p.n_decode > 0) {
        constexpr int LDS = LA_DEC_WAVES * G::TILE;
        static const int rc = la_lds(latent_decode_kernel<RS>, LDS);
        if (rc != OMNI_OK) return rc;
        a.nsplit = p.workspace ? la_splits(p.n_decode, p.heads, p.max_keys) : 1;
        hipLaunchKernelGGL(latent_decode_kernel<RS>, dim3((p.heads + 15) / 16, p.n_decode, a.nsplit), dim3(64 * LA_DEC_WAVES), LDS, st, a);
        OMNI_CHECK_LAUNCH("omni_latent_attn(decode)");
        if (a.nsplit > 1) {
            hipLaunchKernelGGL(latent_merge_kernel, dim3(p.n_decode * p.heads), dim3(64), 0, st, (const float*)a.partial, a.gate, a.out, a.nsplit, p.rp);
            OMNI_CHECK_LAUNCH("omni_latent_attn(merge)");
        }
    }
    if (p.n_tiles > 0) {
        constexpr int PW = 8, LDS = 2 * G::TILE;
        static const int rc = la_lds(latent_prefill_kernel<RS, PW, 8 / PW>, LDS);
        if (rc != OMNI_OK) return rc;
        hipLaunchKernelGGL((latent_prefill_kernel<RS, PW, 8 / PW>), dim3(p.n_tiles), dim3(64 * PW), LDS, st, a);
        OMNI_CHECK_LAUNCH("omni_latent_attn(prefill)");
    }
    return OMNI_OK;
}

extern "C" int omni_latent_attn_run(const omni_latent_attn* pp, void* stream) {
    OMNI_CHECK_ARG(pp && pp->q && pp->cache && pp->out && pp->block_table && pp->row_of_tok && pp->positions, "omni_latent_attn: null pointer");
    const omni_latent_attn& p = *pp;
    OMNI_CHECK_ARG(p.heads > 0 && p.rp > 0 && p.rp % 32 == 0 && p.rp <= LA_PLAIN_MAX, "omni_latent_attn: heads=%d latent width %d (multiple of 32, <= %d)", p.heads, p.rp, LA_PLAIN_MAX);
    OMNI_CHECK_ARG(p.block_size > 0 && (p.block_size & (p.block_size - 1)) == 0 && p.bt_stride > 0, "omni_latent_attn: block_size=%d (a power of two)", p.block_size);
    OMNI_CHECK_ARG(p.n_decode >= 0 && p.n_decode <= p.T && p.n_decode <= 65535 && p.n_tiles >= 0 && (p.n_tiles == 0 || p.tiles) && (p.n_decode == p.T || p.n_tiles > 0 || p.elem == 1),
                   "omni_latent_attn: T=%d n_decode=%d n_tiles=%d", p.T, p.n_decode, p.n_tiles);
    OMNI_CHECK_ARG(!p.workspace || p.workspace_bytes >= omni_latent_attn_workspace_bytes(p.n_decode, p.heads, p.rp), "omni_latent_attn: workspace of %lld bytes", (long long)p.workspace_bytes);
    if (p.T <= 0) return OMNI_OK;
    hipStream_t st = (hipStream_t)stream;
    if (p.elem == 1 || !omni_latent_attn_mfma(p.rp)) {
        const dim3 grid((unsigned)((int64_t)p.T * p.heads)), block(64);
        if (p.elem == 1)
            hipLaunchKernelGGL(latent_plain_kernel<float>, grid, block, 0, st, (const float*)p.q, (const float*)p.cache, p.gate, (float*)p.out, p.block_table, p.bt_stride,
                               p.block_size, p.row_of_tok, p.positions, p.heads, p.rp, p.scale);
        else
            hipLaunchKernelGGL(latent_plain_kernel<uint16_t>, grid, block, 0, st, (const uint16_t*)p.q, (const uint16_t*)p.cache, p.gate, (uint16_t*)p.out, p.block_table,
                               p.bt_stride, p.block_size, p.row_of_tok, p.positions, p.heads, p.rp, p.scale);
        OMNI_CHECK_LAUNCH("omni_latent_attn(plain)");
        return OMNI_OK;
    }
    LatentArgs a{};
    a.q = (const uint16_t*)p.q; a.cache = (const uint16_t*)p.cache; a.gate = p.gate; a.out = (uint16_t*)p.out;
    a.block_table = p.block_table; a.bt_stride = p.bt_stride; a.bs_shift = __builtin_ctz((unsigned)p.block_size); a.bs_mask = p.block_size - 1;
    a.row_of_tok = p.row_of_tok; a.positions = p.positions; a.tiles = p.tiles;
    a.heads = p.heads; a.qs = p.scale * LA_LOG2E; a.partial = p.workspace; a.nsplit = 1;
    switch (p.rp / 32) {
#define X(RS_) case RS_: return la_run<RS_>(p, a, st);
        LA_WIDTHS(X)
#undef X
        default: return OMNI_EINVAL;
    }
}
