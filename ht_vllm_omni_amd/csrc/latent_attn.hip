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
//   latent_decode_kernel   one token: up to 16 heads fill the 16 query rows.  Four waves take one 16-key tile each for the scores, agree on the
//                          row maxima, and share the second product by output columns: no sums to merge across waves at the end.  The
//                          next tiles travel in registers meanwhile.  KV splits leave records a small kernel merges
//   latent_prefill_kernel  tiles of up to la_tile_rows() query rows of one sequence, 16 per wave; the waves share each 32-key tile
//                          (double-buffered, one barrier per tile)
//   latent_plain_kernel    any width, bf16 or fp32: one wave per query row on the vector units (the 32-bit mode)
#include "attn_tile.cuh"
#include "../../include/omni_decoder.h"

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

// scores of one 16-row group against the 32-key tile at `img` (four independent MFMA chains)
template <int RS>
__device__ __forceinline__ void la_scores(const unsigned char* img, const u32x4 (&Q)[RS], int c, int qk, f32x4 (&S)[2]) {
    constexpr int PITCH = LatentGeom<RS>::PITCH;
    f32x4 T[2];
#pragma unroll
    for (int kt = 0; kt < 2; ++kt) S[kt] = T[kt] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < RS; ++s) {
#pragma unroll
        for (int kt = 0; kt < 2; ++kt) {
            const u32x4 A = *reinterpret_cast<const u32x4*>(img + (16 * kt + c) * PITCH + (32 * s + 8 * qk) * 2);
            if (s & 1) T[kt] = mfma16(A, Q[s], T[kt]);
            else S[kt] = mfma16(A, Q[s], S[kt]);
        }
    }
#pragma unroll
    for (int kt = 0; kt < 2; ++kt) S[kt] += T[kt];
}

// this lane's 8 scores of row c in exponent units; returns the row's maximum over the tile.  nlive: keys of the tile the row sees (<= 0: none)
__device__ __forceinline__ float la_row_max(const f32x4 (&S)[2], float qs, int nlive, int qk, float (&sv)[8]) {
    float mx = LA_SENT;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
        const int kidx = (j < 4) ? 4 * qk + j : 16 + 4 * qk + (j - 4);
        sv[j] = S[j >> 2][j & 3] * qs;
        if (kidx < nlive) mx = fmaxf(mx, sv[j]);
    }
    return xor32_max(xor16_max(mx));
}

struct LaWeights { u32x4 hi, mid, lo; };
// weights exp2(sv - m) of the visible keys as three bf16 terms; rs = their sum over the tile
__device__ __forceinline__ LaWeights la_weights(const float (&sv)[8], int nlive, int qk, float m, float& rs) {
    float p[8];
    rs = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
        const int kidx = (j < 4) ? 4 * qk + j : 16 + 4 * qk + (j - 4);
        p[j] = kidx < nlive ? exp2f(sv[j] - m) : 0.f;
        rs += p[j];
    }
    rs = xor32_sum(xor16_sum(rs));
    LaWeights w;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        uint32_t hi, mid, lo;
        split3(p[2 * e], p[2 * e + 1], hi, mid, lo);
        w.hi[e] = hi; w.mid[e] = mid; w.lo[e] = lo;
    }
    return w;
}

// C^T fragment of d tile dt: lane (d = c, qk) gets the 8 keys of its contraction slots
template <int RS>
__device__ __forceinline__ u32x4 la_transposed(const unsigned char* img, int dt, int c, int qk) {
    return la_transposed_at(img, LatentGeom<RS>::PITCH, dt, c, qk);
}

template <int RS>
__global__ __launch_bounds__(64 * LA_DEC_WAVES, 2) void latent_decode_kernel(const LatentArgs a) {
    using G = LatentGeom<RS>;
    constexpr int HALF = 16 * G::PITCH;               // one wave's 16-key image; two waves' images are one 32-key tile of the second product
    constexpr int DPW = (2 * RS + LA_DEC_WAVES - 1) / LA_DEC_WAVES;      // output column tiles of a wave: wave, wave + 4, ...
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];  // [wave] images | [pair][term][lane] weights
    __shared__ float sm[LA_DEC_WAVES][16], sl[LA_DEC_WAVES][16];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int c = lane & 15, qk = lane >> 4;
    const int t = blockIdx.y, split = blockIdx.z;
    const int head = blockIdx.x * 16 + c, hc = min(head, a.heads - 1);
    constexpr int rp = RS * 32;
    unsigned char* img = lds + wave * HALF;
    u32x4* pw = reinterpret_cast<u32x4*>(lds + LA_DEC_WAVES * HALF);
    const int len = a.positions[t] + 1;
    const int32_t* bt = a.block_table + (size_t)a.row_of_tok[t] * a.bt_stride;
    const int ntiles = (len + 15) / 16;
    const int nsplit = la_row_splits(ntiles, a.nsplit);
    if (split >= nsplit) return;
    const int t0 = (int)((long long)ntiles * split / nsplit), t1 = (int)((long long)ntiles * (split + 1) / nsplit);
    const int end = min(len, t1 * 16);                // keys of this split
    u32x4 st[RS];                                     // the wave's next tile on its way to LDS (16 rows = RS 16-byte loads per lane)
    auto block_of = [&](int tile) { return bt[min(tile * 16 + c, len - 1) >> a.bs_shift]; };
    auto fetch = [&](int tile, int blk) {
        const int key = min(tile * 16 + c, len - 1);  // keys past the end: a valid row, masked below
        const int slot = (blk << a.bs_shift) + (key & a.bs_mask);
#pragma unroll
        for (int j = 0; j < RS; ++j) {
            const int i = lane + 64 * j;
            const int kk = i / G::CH, ch = i - kk * G::CH;
            const int row = G::CH % 64 == 0 ? __builtin_amdgcn_readlane(slot, j / (G::CH / 64 > 0 ? G::CH / 64 : 1)) : __shfl(slot, kk, 64);
            st[j] = ld16_nt(a.cache + (size_t)row * rp + ch * 8);
        }
    };
    int blk = 0;                                      // block ids are looked up a round ahead of the rows
    if (t0 < t1) {
        blk = block_of(t0 + wave);
        fetch(t0 + wave, blk);
        blk = block_of(t0 + wave + LA_DEC_WAVES);
    }
    u32x4 Q[RS];
#pragma unroll
    for (int s = 0; s < RS; ++s) Q[s] = ld16(a.q + ((size_t)t * a.heads + hc) * rp + 32 * s + 8 * qk);
    f32x4 O[DPW];
#pragma unroll
    for (int i = 0; i < DPW; ++i) O[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
    float m = LA_SENT, l = 0.f;                       // m: common to the waves; l: this wave's keys
    for (int base = t0; base < t1; base += LA_DEC_WAVES) {
        const int key0 = (base + wave) * 16 + 4 * qk; // the lane's keys: key0 .. key0 + 3
#pragma unroll
        for (int j = 0; j < RS; ++j) {
            const int i = lane + 64 * j;
            const int kk = i / G::CH, ch = i - kk * G::CH;
            *reinterpret_cast<u32x4*>(img + kk * G::PITCH + ch * 16) = st[j];
        }
        if (base + LA_DEC_WAVES < t1) {
            fetch(base + wave + LA_DEC_WAVES, blk);
            blk = block_of(base + wave + 2 * LA_DEC_WAVES);
        }
        __builtin_amdgcn_wave_barrier();
        f32x4 S4[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) S4[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
        constexpr int AB = RS < 8 ? RS : 8;           // operand reads in flight
#pragma unroll
        for (int s0 = 0; s0 < RS; s0 += AB) {
            u32x4 A[AB];
#pragma unroll
            for (int s = 0; s < AB; ++s)
                if (s0 + s < RS) A[s] = *reinterpret_cast<const u32x4*>(img + c * G::PITCH + (32 * (s0 + s) + 8 * qk) * 2);
#pragma unroll
            for (int s = 0; s < AB; ++s)
                if (s0 + s < RS) S4[s & 3] = mfma16(A[s], Q[s0 + s], S4[s & 3]);
        }
        const f32x4 S = (S4[0] + S4[1]) + (S4[2] + S4[3]);
        float sv[4], mx = LA_SENT;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            sv[j] = S[j] * a.qs;
            if (key0 + j < end) mx = fmaxf(mx, sv[j]);
        }
        mx = xor32_max(xor16_max(mx));
        if (qk == 0) sm[wave][c] = mx;
        __syncthreads();                              // maxima and images of this round
        float mn = m;
#pragma unroll
        for (int w = 0; w < LA_DEC_WAVES; ++w) mn = fmaxf(mn, sm[w][c]);
        const float alpha = exp2f(m - mn);            // both the sentinel: 1, harmless (l = 0, O = 0)
        m = mn;
        float p[4], rs = 0.f;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            p[j] = key0 + j < end ? exp2f(sv[j] - m) : 0.f;
            rs += p[j];
        }
        l = l * alpha + xor32_sum(xor16_sum(rs));
        u32x2 w3[3];                                  // three bf16 terms whose sum is the fp32 weight
#pragma unroll
        for (int e = 0; e < 2; ++e) {
            uint32_t hi, mid, lo;
            split3(p[2 * e], p[2 * e + 1], hi, mid, lo);
            w3[0][e] = hi; w3[1][e] = mid; w3[2][e] = lo;
        }
#pragma unroll
        for (int i = 0; i < 3; ++i) reinterpret_cast<u32x2*>(pw + ((wave >> 1) * 3 + i) * 64 + lane)[wave & 1] = w3[i];
#pragma unroll
        for (int i = 0; i < DPW; ++i) O[i] *= alpha;
        __syncthreads();                              // weights of this round
#pragma unroll
        for (int u = 0; u < LA_DEC_WAVES / 2; ++u) {
            if (base + 2 * u >= t1) break;            // (uniform; an image past t1 inside a pair holds valid rows with zero weights)
            u32x4 W[3], VT[DPW];
#pragma unroll
            for (int i = 0; i < 3; ++i) W[i] = pw[(u * 3 + i) * 64 + lane];
#pragma unroll
            for (int i = 0; i < DPW; ++i) VT[i] = la_transposed<RS>(lds + u * 2 * HALF, min(wave + LA_DEC_WAVES * i, 2 * RS - 1), c, qk);
#pragma unroll
            for (int k = 2; k >= 0; --k)
#pragma unroll
                for (int i = 0; i < DPW; ++i) O[i] = mfma16(VT[i], W[k], O[i]);
        }
        if (base + LA_DEC_WAVES < t1) __syncthreads();      // the images are rewritten by the next round
    }
    if (qk == 0) sl[wave][c] = l;
    __syncthreads();
    float L = 0.f;
#pragma unroll
    for (int w = 0; w < LA_DEC_WAVES; ++w) L += sl[w][c];
    if (head >= a.heads) return;
    const size_t rh = (size_t)t * a.heads + head;
    float* rec = nsplit > 1 ? a.partial + (rh * a.nsplit + split) * (rp + 4) : nullptr;
    if (rec && wave == 0 && qk == 0) { rec[0] = m; rec[1] = L; }
    const float inv = (L > 0.f ? 1.0f / L : 0.f) * (a.gate ? a.gate[rh] : 1.0f);
#pragma unroll
    for (int i = 0; i < DPW; ++i) {
        const int d = wave + LA_DEC_WAVES * i;
        if (d >= 2 * RS) continue;
        if (rec) {
            *reinterpret_cast<f32x4*>(rec + 4 + 16 * d + 4 * qk) = O[i];
        } else {
            const f32x4 v = O[i] * inv;
            *reinterpret_cast<uint2*>(a.out + rh * rp + 16 * d + 4 * qk) = make_uint2(pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3]));
        }
    }
}

// KV splits of one (token, head): lane s holds split s's weight, every thread 4 columns
__global__ __launch_bounds__(128) void latent_merge_kernel(const float* __restrict__ partial, const float* __restrict__ gate, uint16_t* __restrict__ out,
                                                           const int32_t* __restrict__ positions, int heads, int max_split, int rp) {
    const size_t rh = blockIdx.x;
    const int nsplit = la_row_splits((positions[rh / heads] + 16) / 16, max_split);
    if (nsplit == 1) return;                           // the decode kernel wrote the row
    const float* base = partial + rh * max_split * (rp + 4);
    const int lane = threadIdx.x & 63, k = threadIdx.x * 4;
    const float2 ml = lane < nsplit ? *reinterpret_cast<const float2*>(base + (size_t)lane * (rp + 4)) : make_float2(LA_SENT, 0.f);
    const float M = wave_max(ml.x);
    const float w = lane < nsplit ? exp2f(ml.x - M) : 0.f;
    const float L = wave_sum(ml.y * w);
    if (k >= rp) return;
    f32x4 v = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int s = 0; s < nsplit; ++s)
        v += *reinterpret_cast<const f32x4*>(base + (size_t)s * (rp + 4) + 4 + k) * __int_as_float(__builtin_amdgcn_readlane(__float_as_int(w), s));
    v *= (L > 0.f ? 1.0f / L : 0.f) * (gate ? gate[rh] : 1.0f);
    *reinterpret_cast<uint2*>(out + rh * rp + k) = make_uint2(pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3]));
}

template <int RS, int PW>
__global__ __launch_bounds__(64 * PW, 2) void latent_prefill_kernel(const LatentArgs a) {
    using G = LatentGeom<RS>;
    constexpr int NT = 64 * PW, ITEMS = LA_KEYS * G::CH, LOADS = (ITEMS + NT - 1) / NT;
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];      // two tile images
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int c = lane & 15, qk = lane >> 4;
    const int row0 = a.tiles[2 * blockIdx.x], nrows = a.tiles[2 * blockIdx.x + 1];
    constexpr int rp = RS * 32;
    const int32_t* bt = a.block_table + (size_t)a.row_of_tok[row0 / a.heads] * a.bt_stride;
    const int r = wave * 16 + c;
    const size_t frow = (size_t)(row0 + min(r, nrows - 1));
    const int see = r < nrows ? a.positions[frow / a.heads] + 1 : 0;         // keys the row sees
    const int wsee = wave * 16 < nrows ? a.positions[(row0 + min(wave * 16 + 15, nrows - 1)) / a.heads] + 1 : 0;      // most keys of the wave's rows
    const int nkeys = a.positions[(row0 + nrows - 1) / a.heads] + 1;
    u32x4 Q[RS];
    f32x4 O[2 * RS];
#pragma unroll
    for (int s = 0; s < RS; ++s) Q[s] = ld16(a.q + frow * rp + 32 * s + 8 * qk);
#pragma unroll
    for (int d = 0; d < 2 * RS; ++d) O[d] = (f32x4){0.f, 0.f, 0.f, 0.f};
    float m = LA_SENT, l = 0.f;
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
        f32x4 S[2];
        la_scores<RS>(img, Q, c, qk, S);
        float sv[8], rs;
        const float mn = fmaxf(m, la_row_max(S, a.qs, see - k0, qk, sv));
        const float alpha = exp2f(m - mn);              // both the sentinel: 1, harmless (l = 0, O = 0)
        m = mn;
        const LaWeights w = la_weights(sv, see - k0, qk, mn, rs);
        l = l * alpha + rs;
        if (__any(alpha != 1.0f)) {
#pragma unroll
            for (int d = 0; d < 2 * RS; ++d) O[d] *= alpha;
        }
#pragma unroll
        for (int d0 = 0; d0 < 2 * RS; d0 += 2) {        // pairs of column tiles: independent chains between dependent MFMAs
            u32x4 VT[2];
#pragma unroll
            for (int d = 0; d < 2; ++d) VT[d] = la_transposed<RS>(img, d0 + d, c, qk);
#pragma unroll
            for (int d = 0; d < 2; ++d) O[d0 + d] = mfma16(VT[d], w.lo, O[d0 + d]);
#pragma unroll
            for (int d = 0; d < 2; ++d) O[d0 + d] = mfma16(VT[d], w.mid, O[d0 + d]);
#pragma unroll
            for (int d = 0; d < 2; ++d) O[d0 + d] = mfma16(VT[d], w.hi, O[d0 + d]);
        }
    }
    if (see <= 0) return;
    const float inv = 1.0f / l * (a.gate ? a.gate[frow] : 1.0f);
#pragma unroll
    for (int d = 0; d < 2 * RS; ++d) {
        const f32x4 v = O[d] * inv;
        *reinterpret_cast<uint2*>(a.out + frow * rp + 16 * d + 4 * qk) = make_uint2(pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3]));
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
// query rows per prompt work item.  Measured (16 heads, 1 x 2048 / 16 x 128 / 4 x 2048 tokens): width 512 by 128 rows 277 / 36 / 652 us, by 64 307 / 42 /
// 750; width 256 by 128 rows 162 / 22 / 370, by 64 -- two workgroups fit a CU -- 129 / 18 / 340
static constexpr int la_tile_rows(int rp) { return rp > 256 ? 128 : 64; }
extern "C" int omni_latent_attn_tile_rows(int rp) { return la_tile_rows(rp); }

static int la_splits(int n_decode, int heads, int max_keys) { return la_split_count(n_decode * ((heads + 15) / 16), max_keys); }

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
    if (bytes <= 60 * 1024) return OMNI_OK;         // (static shared memory comes on top)
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, bytes);
    if (e != hipSuccess) { omni_set_error("omni_latent_attn: LDS attribute: %s", hipGetErrorString(e)); return OMNI_EHIP; }
    return OMNI_OK;
}

template <int RS>
static int la_run(const omni_latent_attn& p, LatentArgs a, hipStream_t st) {
    using G = LatentGeom<RS>;
    if (p.n_decode > 0) {
        constexpr int LDS = LA_DEC_WAVES * 16 * G::PITCH + LA_DEC_WAVES / 2 * 3 * 1024;
        static const int rc = la_lds(latent_decode_kernel<RS>, LDS);
        if (rc != OMNI_OK) return rc;
        a.nsplit = p.workspace ? la_splits(p.n_decode, p.heads, p.max_keys) : 1;
        hipLaunchKernelGGL(latent_decode_kernel<RS>, dim3((p.heads + 15) / 16, p.n_decode, a.nsplit), dim3(64 * LA_DEC_WAVES), LDS, st, a);
        OMNI_CHECK_LAUNCH("omni_latent_attn(decode)");
        if (a.nsplit > 1) {
            hipLaunchKernelGGL(latent_merge_kernel, dim3(p.n_decode * p.heads), dim3(p.rp > 256 ? 128 : 64), 0, st, (const float*)a.partial, a.gate, a.out, a.positions, p.heads, a.nsplit, p.rp);
            OMNI_CHECK_LAUNCH("omni_latent_attn(merge)");
        }
    }
    if (p.n_tiles > 0) {
        constexpr int PW = la_tile_rows(RS * 32) / 16, LDS = 2 * G::TILE;
        static const int rc = la_lds(latent_prefill_kernel<RS, PW>, LDS);
        if (rc != OMNI_OK) return rc;
        hipLaunchKernelGGL((latent_prefill_kernel<RS, PW>), dim3(p.n_tiles), dim3(64 * PW), LDS, st, a);
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
    OMNI_CHECK_ARG(p.n_tiles == 0 || p.tile_rows == la_tile_rows(p.rp), "omni_latent_attn: tile_rows=%d (omni_latent_attn_tile_rows(%d) = %d)", p.tile_rows, p.rp, la_tile_rows(p.rp));
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
