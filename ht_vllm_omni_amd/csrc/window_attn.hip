// Causal grouped attention over a paged cache of keys and values, with an optional sliding window and an optional number per head in the softmax's
// denominator (include/omni_decoder.h omni_window_attn).  The heads that share a key / value head are query rows of one matrix problem, as all
// heads are in latent_attn.hip; the transposed-operand scheme and the three-term weights are the same (attn_tile.cuh):
//   S^T[key][row] = K . Q^T      A = K (lane (key, chunk qk): 8 dims), B = Q^T (registers for the whole kernel)
//   O^T[d][row]  += V^T . P^T    A = V^T: ds_read_b64_tr_b16 out of the row-major tile
// Scores, softmax statistics and weights are fp32.  Widths are run-time (dp, vp multiples of 32) below a compile-time bound WS; EX: both equal it.
//
//   window_decode_kernel   one token and one key / value head: up to 16 query heads fill the 16 rows.  Four waves score one 16-key tile each -- keys go
//                          from HBM straight into MFMA operands -- agree on the row maxima and share the second product by output columns.  Walks
//                          the window's tiles only; KV splits leave records a small kernel merges
//   window_prefill_kernel  up to wa_tile_rows() query rows (tokens x grouped heads) of one sequence, 16 per wave; the waves share each 32-key tile
//   window_plain_kernel    any width, bf16 or fp32: one wave per (token, head) on the vector units (the 32-bit mode)
#include "attn_tile.cuh"
#include "../../include/omni_decoder.h"

struct WinArgs {
    const uint16_t* q; const uint16_t* kc; const uint16_t* vc; const uint16_t* gate; const float* sink; uint16_t* out; int frag;
    const int32_t* block_table; int bt_stride, bs_shift, bs_mask;
    const int32_t* row_of_tok; const int32_t* positions; const int32_t* tiles;
    int heads, kv_heads, rep;       // rep = heads / kv_heads
    int ds, vs;                     // dp / 32, vp / 32
    float qs; int window;           // scale * log2(e); INT_MAX: no window
    float* partial; int nsplit;
};

// first key a token at `pos` sees
__device__ __forceinline__ int wa_first(int pos, int window) { return max(0, pos - window + 1); }

// 4 output columns [k, k + 4) of a token's row, times the gate
__device__ __forceinline__ void wa_store(const uint16_t* gate, uint16_t* out, int frag, size_t t, int k, int width, f32x4 v) {
    if (gate) {
        const uint2 g = *reinterpret_cast<const uint2*>(gate + t * width + k);
        v[0] *= bf_lo(g.x); v[1] *= bf_hi(g.x); v[2] *= bf_lo(g.y); v[3] *= bf_hi(g.y);
    }
    *reinterpret_cast<uint2*>(out + (frag ? frag_off((int)t, k, width) : t * width + k)) = make_uint2(pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3]));
}

template <int WS, bool EX>
__global__ __launch_bounds__(64 * LA_DEC_WAVES, 2) void window_decode_kernel(const WinArgs a) {
    constexpr int DPW = (2 * WS + LA_DEC_WAVES - 1) / LA_DEC_WAVES;      // output column tiles of a wave: wave, wave + 4, ...
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];  // [wave] 16-key images of V | [pair][term][lane] weights
    __shared__ float sm[LA_DEC_WAVES][16], sl[LA_DEC_WAVES][16];
    const int ds = EX ? WS : a.ds, vs = EX ? WS : a.vs, dp = ds * 32, vp = vs * 32;
    const int pitch = vp * 2 + 32, himg = 16 * pitch;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int c = lane & 15, qk = lane >> 4;
    const int t = blockIdx.y, split = blockIdx.z;
    const int rt = (a.rep + 15) >> 4, g = blockIdx.x / rt;
    const int hr = (blockIdx.x - g * rt) * 16 + c, head = g * a.rep + min(hr, a.rep - 1);
    unsigned char* img = lds + wave * himg;
    u32x4* pw = reinterpret_cast<u32x4*>(lds + LA_DEC_WAVES * himg);
    const int pos = a.positions[t], len = pos + 1, lo = wa_first(pos, a.window);
    const int32_t* bt = a.block_table + (size_t)a.row_of_tok[t] * a.bt_stride;
    const int tl = lo >> 4, ntiles = (len + 15) / 16 - tl;
    const int nsplit = la_row_splits(ntiles, a.nsplit);
    if (split >= nsplit) return;
    const int t0 = tl + (int)((long long)ntiles * split / nsplit), t1 = tl + (int)((long long)ntiles * (split + 1) / nsplit);
    const int end = min(len, t1 * 16);                // keys of this split: [lo, end) from tile t0 on
    u32x4 K[WS], st[WS];                              // the wave's next tile: keys as operands, values on their way to LDS
    auto block_of = [&](int tile) { return bt[min(tile * 16 + c, len - 1) >> a.bs_shift]; };
    auto fetch = [&](int tile, int blk) {             // lane (c, qk): 16-byte pieces qk, qk + 4, ... of key c's rows
        const int key = min(tile * 16 + c, len - 1);  // keys past the end: a valid row, masked below
        const size_t row = ((size_t)(blk * a.kv_heads + g) << a.bs_shift) + (key & a.bs_mask);
#pragma unroll
        for (int s = 0; s < WS; ++s)
            if (EX || s < ds) K[s] = ld16_nt(a.kc + row * dp + 32 * s + 8 * qk);
#pragma unroll
        for (int s = 0; s < WS; ++s)
            if (EX || s < vs) st[s] = ld16_nt(a.vc + row * vp + 32 * s + 8 * qk);
    };
    int blk = block_of(t0 + wave);                    // block ids are looked up a round ahead of the rows
    fetch(t0 + wave, blk);
    blk = block_of(t0 + wave + LA_DEC_WAVES);
    u32x4 Q[WS];
#pragma unroll
    for (int s = 0; s < WS; ++s)
        if (EX || s < ds) Q[s] = ld16(a.q + ((size_t)t * a.heads + head) * dp + 32 * s + 8 * qk);
    f32x4 O[DPW];
#pragma unroll
    for (int i = 0; i < DPW; ++i) O[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
    // m: common to the waves; l: this wave's keys.  The sink is a key without a value: it opens the first split's statistics
    const bool sink = a.sink && split == 0;
    float m = sink ? a.sink[head] * LA_LOG2E : LA_SENT, l = sink && wave == 0 ? 1.f : 0.f;
    for (int base = t0; base < t1; base += LA_DEC_WAVES) {
        const int key0 = (base + wave) * 16 + 4 * qk; // the lane's keys: key0 .. key0 + 3
#pragma unroll
        for (int s = 0; s < WS; ++s)
            if (EX || s < vs) *reinterpret_cast<u32x4*>(img + c * pitch + (32 * s + 8 * qk) * 2) = st[s];
        f32x4 S2[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
        for (int s = 0; s < WS; ++s)
            if (EX || s < ds) S2[s & 1] = mfma16(K[s], Q[s], S2[s & 1]);
        if (base + LA_DEC_WAVES < t1) {
            fetch(base + wave + LA_DEC_WAVES, blk);
            blk = block_of(base + wave + 2 * LA_DEC_WAVES);
        }
        const f32x4 S = S2[0] + S2[1];
        float sv[4], mx = LA_SENT;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            sv[j] = S[j] * a.qs;
            if (key0 + j >= lo && key0 + j < end) mx = fmaxf(mx, sv[j]);
        }
        mx = xor32_max(xor16_max(mx));
        if (qk == 0) sm[wave][c] = mx;
        __syncthreads();                              // maxima and images of this round
        float mn = m;
#pragma unroll
        for (int w = 0; w < LA_DEC_WAVES; ++w) mn = fmaxf(mn, sm[w][c]);
        const float alpha = exp2_w(m - mn);            // both the sentinel: 1, harmless (l = 0, O = 0)
        m = mn;
        float p[4], rs = 0.f;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            p[j] = key0 + j >= lo && key0 + j < end ? exp2_w(sv[j] - m) : 0.f;
            rs += p[j];
        }
        l = l * alpha + xor32_sum(xor16_sum(rs));
        u32x2 w3[3];                                  // three bf16 terms whose sum is the fp32 weight
#pragma unroll
        for (int e = 0; e < 2; ++e) {
            uint32_t hi, mid, low;
            split3(p[2 * e], p[2 * e + 1], hi, mid, low);
            w3[0][e] = hi; w3[1][e] = mid; w3[2][e] = low;
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
            for (int i = 0; i < DPW; ++i) VT[i] = la_transposed_at(lds + u * 2 * himg, pitch, min(wave + LA_DEC_WAVES * i, 2 * vs - 1), c, qk);
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
    if (hr >= a.rep) return;
    float* rec = nsplit > 1 ? a.partial + (((size_t)t * a.heads + head) * a.nsplit + split) * (vp + 4) : nullptr;
    if (rec && wave == 0 && qk == 0) { rec[0] = m; rec[1] = L; }
    const float inv = L > 0.f ? 1.0f / L : 0.f;
#pragma unroll
    for (int i = 0; i < DPW; ++i) {
        const int d = wave + LA_DEC_WAVES * i;
        if (d >= 2 * vs) continue;
        if (rec) *reinterpret_cast<f32x4*>(rec + 4 + 16 * d + 4 * qk) = O[i];
        else wa_store(a.gate, a.out, a.frag, t, head * vp + 16 * d + 4 * qk, a.heads * vp, O[i] * inv);
    }
}

// KV splits of one (token, head): lane s holds split s's weight, every thread 4 columns
__global__ __launch_bounds__(64) void window_merge_kernel(const WinArgs a, int max_split) {
    const size_t rh = blockIdx.x;
    const int t = (int)(rh / a.heads), head = (int)(rh - (size_t)t * a.heads), vp = a.vs * 32;
    const int pos = a.positions[t];
    const int nsplit = la_row_splits((pos + 16) / 16 - (wa_first(pos, a.window) >> 4), max_split);
    if (nsplit == 1) return;                           // the decode kernel wrote the row
    const float* base = a.partial + rh * max_split * (vp + 4);
    const int lane = threadIdx.x, k = lane * 4;
    const float2 ml = lane < nsplit ? *reinterpret_cast<const float2*>(base + (size_t)lane * (vp + 4)) : make_float2(LA_SENT, 0.f);
    const float M = wave_max(ml.x);
    const float w = lane < nsplit ? exp2_w(ml.x - M) : 0.f;
    const float L = wave_sum(ml.y * w);
    if (k >= vp) return;
    f32x4 v = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int s = 0; s < nsplit; ++s)
        v += *reinterpret_cast<const f32x4*>(base + (size_t)s * (vp + 4) + 4 + k) * __int_as_float(__builtin_amdgcn_readlane(__float_as_int(w), s));
    wa_store(a.gate, a.out, a.frag, t, head * vp + k, a.heads * vp, v * (L > 0.f ? 1.0f / L : 0.f));
}

template <int WS, bool EX, int PW>
__global__ __launch_bounds__(64 * PW, 2) void window_prefill_kernel(const WinArgs a) {
    constexpr int SPT = PW / 2, LOADS = (WS + SPT - 1) / SPT;                // 32-wide pieces of a row the workgroup loads per pass, passes
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];      // two images of [32 keys | 32 values]
    const int ds = EX ? WS : a.ds, vs = EX ? WS : a.vs, dp = ds * 32, vp = vs * 32;
    const int kpitch = dp * 2 + 32, vpitch = vp * 2 + 32, image = LA_KEYS * (kpitch + vpitch);
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int c = lane & 15, qk = lane >> 4;
    const int row0 = a.tiles[2 * blockIdx.x], nrows = a.tiles[2 * blockIdx.x + 1], g = blockIdx.y;
    const int tok0 = row0 / a.rep;
    const int32_t* bt = a.block_table + (size_t)a.row_of_tok[tok0] * a.bt_stride;
    const int r = wave * 16 + c;
    const int frow = row0 + min(r, nrows - 1), tok = frow / a.rep, head = g * a.rep + frow - tok * a.rep;
    const int pos = a.positions[tok];
    const int hi = r < nrows ? pos + 1 : 0, lo = wa_first(pos, a.window);    // keys the row sees: [lo, hi)
    // keys the wave's rows see, and the tile's: positions grow along the rows
    const bool any = wave * 16 < nrows;
    const int whi = any ? a.positions[(row0 + min(wave * 16 + 15, nrows - 1)) / a.rep] + 1 : 0;
    const int wlo = any ? wa_first(a.positions[(row0 + wave * 16) / a.rep], a.window) : 0;
    // ... and the keys every one of the wave's rows sees: no masks in a tile inside
    const int fhi = wave * 16 + 16 <= nrows ? a.positions[(row0 + wave * 16) / a.rep] + 1 : 0, flo = wa_first(whi - 1, a.window);
    const int nkeys = a.positions[(row0 + nrows - 1) / a.rep] + 1;
    const int kbeg = wa_first(a.positions[tok0], a.window) & ~(LA_KEYS - 1);
    u32x4 Q[WS];
    f32x4 O[2 * WS];
#pragma unroll
    for (int s = 0; s < WS; ++s)
        if (EX || s < ds) Q[s] = ld16(a.q + ((size_t)tok * a.heads + head) * dp + 32 * s + 8 * qk);
#pragma unroll
    for (int d = 0; d < 2 * WS; ++d) O[d] = (f32x4){0.f, 0.f, 0.f, 0.f};
    float m = LA_SENT, l = 0.f;
    if (a.sink) { m = a.sink[head] * LA_LOG2E; l = 1.f; }
    // loader: thread -> key (tid / 4) % 32, 16-byte quarter tid % 4 of the 32-wide pieces tid / 128, + SPT, ...
    const int lkey = (threadIdx.x >> 2) & 31, lq = threadIdx.x & 3, lp = threadIdx.x >> 7;
    u32x4 sk[LOADS], sv_[LOADS];
    auto block_of = [&](int k0) { return bt[min(k0 + lkey, nkeys - 1) >> a.bs_shift]; };
    auto fetch = [&](int k0, int blk) {
        const int key = min(k0 + lkey, nkeys - 1);
        const size_t row = ((size_t)(blk * a.kv_heads + g) << a.bs_shift) + (key & a.bs_mask);
#pragma unroll
        for (int j = 0; j < LOADS; ++j) {
            const int s = lp + SPT * j;
            if (s < ds) sk[j] = ld16(a.kc + row * dp + 32 * s + 8 * lq);
            if (s < vs) sv_[j] = ld16(a.vc + row * vp + 32 * s + 8 * lq);
        }
    };
    int blk = block_of(kbeg);                         // block ids are looked up a tile ahead of the rows
    fetch(kbeg, blk);
    blk = block_of(kbeg + LA_KEYS);
    int buf = 0;
    for (int k0 = kbeg; k0 < nkeys; k0 += LA_KEYS, buf ^= 1) {
        unsigned char* kimg = lds + buf * image;
        unsigned char* vimg = kimg + LA_KEYS * kpitch;
#pragma unroll
        for (int j = 0; j < LOADS; ++j) {
            const int s = lp + SPT * j;
            if (s < ds) *reinterpret_cast<u32x4*>(kimg + lkey * kpitch + (32 * s + 8 * lq) * 2) = sk[j];
            if (s < vs) *reinterpret_cast<u32x4*>(vimg + lkey * vpitch + (32 * s + 8 * lq) * 2) = sv_[j];
        }
        if (k0 + LA_KEYS < nkeys) {
            fetch(k0 + LA_KEYS, blk);
            blk = block_of(k0 + 2 * LA_KEYS);
        }
        __syncthreads();                                // image `buf` complete; image `buf ^ 1` is rewritten only behind the NEXT barrier's arrivals
        if (k0 >= whi || k0 + LA_KEYS <= wlo) continue; // (wave-uniform; the barriers above stay common)
        f32x4 S[2], T[2];
#pragma unroll
        for (int kt = 0; kt < 2; ++kt) S[kt] = T[kt] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < WS; ++s) {
            if (!EX && s >= ds) continue;
#pragma unroll
            for (int kt = 0; kt < 2; ++kt) {
                const u32x4 A = *reinterpret_cast<const u32x4*>(kimg + (16 * kt + c) * kpitch + (32 * s + 8 * qk) * 2);
                if (s & 1) T[kt] = mfma16(A, Q[s], T[kt]);
                else S[kt] = mfma16(A, Q[s], S[kt]);
            }
        }
        float p[8], mx = LA_SENT, rs = 0.f;
        const bool inside = k0 >= flo && k0 + LA_KEYS <= fhi;      // (wave-uniform)
#pragma unroll
        for (int j = 0; j < 8; ++j) p[j] = (S[j >> 2][j & 3] + T[j >> 2][j & 3]) * a.qs;
        if (!inside) {
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                const int key = k0 + la_slot(qk, j);
                if (key < lo || key >= hi) p[j] = -INFINITY;       // a weight of zero against any finite maximum
            }
        }
#pragma unroll
        for (int j = 0; j < 8; ++j) mx = fmaxf(mx, p[j]);
        const float mn = fmaxf(m, xor32_max(xor16_max(mx)));       // (never below the finite sentinel)
        const float alpha = exp2_w(m - mn);              // both the sentinel: 1, harmless (l = 0, O = 0)
        m = mn;
        u32x4 w3[3];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            p[j] = exp2_w(p[j] - mn);
            rs += p[j];
        }
        l = l * alpha + xor32_sum(xor16_sum(rs));
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            uint32_t h0, m0, l0;
            split3(p[2 * e], p[2 * e + 1], h0, m0, l0);
            w3[0][e] = h0; w3[1][e] = m0; w3[2][e] = l0;
        }
        if (__any(alpha != 1.0f)) {
#pragma unroll
            for (int d = 0; d < 2 * WS; ++d) O[d] *= alpha;
        }
#pragma unroll
        for (int d0 = 0; d0 < 2 * WS; d0 += 2) {        // pairs of column tiles: independent chains between dependent MFMAs
            if (!EX && d0 >= 2 * vs) continue;
            u32x4 VT[2];
#pragma unroll
            for (int d = 0; d < 2; ++d) VT[d] = la_transposed_at(vimg, vpitch, d0 + d, c, qk);
#pragma unroll
            for (int k = 2; k >= 0; --k)
#pragma unroll
                for (int d = 0; d < 2; ++d) O[d0 + d] = mfma16(VT[d], w3[k], O[d0 + d]);
        }
    }
    if (r >= nrows) return;
    const float inv = 1.0f / l;
#pragma unroll
    for (int d = 0; d < 2 * WS; ++d)
        if (EX || d < 2 * vs) wa_store(a.gate, a.out, a.frag, tok, head * vp + 16 * d + 4 * qk, a.heads * vp, O[d] * inv);
}

// ---- any width, bf16 or fp32 elements: one wave per (token, head), 64 keys per pass (lane = key for the scores, lane = dims for the sum)
template <typename E>
__device__ __forceinline__ float wa_ld(const E* p, size_t i) {
    if constexpr (sizeof(E) == 4) return p[i];
    else return bf2f(p[i]);
}

#define WA_PLAIN_MAX 1024
template <typename E>
__global__ __launch_bounds__(64) void window_plain_kernel(const omni_window_attn a, int window) {
    __shared__ float sq[WA_PLAIN_MAX], sp[64];
    __shared__ size_t srow[64];
    constexpr int NI = WA_PLAIN_MAX / 64;
    const E* q = (const E*)a.q;
    const E* kc = (const E*)a.kc;
    const E* vc = (const E*)a.vc;
    const int lane = threadIdx.x, rep = a.heads / a.kv_heads;
    const size_t rh = blockIdx.x;
    const int t = (int)(rh / a.heads), head = (int)(rh - (size_t)t * a.heads), g = head / rep;
    for (int k = lane; k < a.dp; k += 64) sq[k] = wa_ld(q, rh * a.dp + k);
    const int pos = a.positions[t], len = pos + 1, lo = wa_first(pos, window);
    const int32_t* bt = a.block_table + (size_t)a.row_of_tok[t] * a.bt_stride;
    float m = LA_SENT, l = 0.f, acc[NI];
    if (a.sink) { m = a.sink[head]; l = 1.f; }
#pragma unroll
    for (int i = 0; i < NI; ++i) acc[i] = 0.f;
    for (int k0 = lo; k0 < len; k0 += 64) {
        __syncthreads();                               // one wave per workgroup: orders the LDS traffic of the passes
        const int key = k0 + lane, kk = min(key, len - 1);
        const size_t row = ((size_t)bt[kk / a.block_size] * a.kv_heads + g) * a.block_size + kk % a.block_size;
        float s = 0.f;
        for (int k = 0; k < a.dp; ++k) s = fmaf(sq[k], wa_ld(kc, row * a.dp + k), s);
        s *= a.scale;
        const bool ok = key < len;
        const float mn = fmaxf(m, wave_max(ok ? s : LA_SENT));
        const float alpha = expf(m - mn), p = ok ? expf(s - mn) : 0.f;
        l = l * alpha + wave_sum(p);
        m = mn;
        sp[lane] = p;
        srow[lane] = row;
        __syncthreads();
        const int nk = min(64, len - k0);
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            const int d = lane + 64 * i;
            if (d >= a.vp) continue;
            float v = acc[i] * alpha;
            for (int u = 0; u < nk; ++u) v = fmaf(sp[u], wa_ld(vc, srow[u] * a.vp + d), v);
            acc[i] = v;
        }
    }
    const float inv = 1.0f / l;
    const int width = a.heads * a.vp;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
        const int d = lane + 64 * i;
        if (d >= a.vp) continue;
        const int k = head * a.vp + d;
        const float v = acc[i] * inv * (a.gate ? wa_ld((const E*)a.gate, (size_t)t * width + k) : 1.0f);
        E* o = (E*)a.out + (a.frag ? frag_off(t, k, width) : (size_t)t * width + k);
        if constexpr (sizeof(E) == 4) *o = v;
        else *o = f2bf(v);
    }
}

// ---- host side
// compile-time width bound of the matrix-core kernels: 2, 4 or 8 (times 32); 0: too wide, the plain kernel runs
static int wa_bound(int dp, int vp) {
    const int w = (dp > vp ? dp : vp) / 32;
    return w <= 2 ? 2 : (w <= 4 ? 4 : (w <= 8 ? 8 : 0));
}
// (measured, 16 heads over 4 of 128, window 1024, 4 x 2048 tokens: 128 rows 174 us, 64 rows 191; 1 x 2048: 60 / 61)
static constexpr int wa_rows_of(int ws) { return ws <= 4 ? 128 : 64; }
extern "C" int omni_window_attn_tile_rows(int dp, int vp) {
    const int w = wa_bound(dp, vp);
    return w ? wa_rows_of(w) : 64;
}

extern "C" int64_t omni_window_attn_workspace_bytes(int n_decode, int heads, int vp) {
    return (int64_t)n_decode * heads * LA_MAX_SPLIT * (vp + 4) * (int64_t)sizeof(float);
}

template <typename K>
static int wa_lds(K kernel, int bytes) {
    if (bytes <= 60 * 1024) return OMNI_OK;         // (static shared memory comes on top)
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, bytes);
    if (e != hipSuccess) { omni_set_error("omni_window_attn: LDS attribute: %s", hipGetErrorString(e)); return OMNI_EHIP; }
    return OMNI_OK;
}

template <int WS, bool EX>
static int wa_run(const omni_window_attn& p, WinArgs a, hipStream_t st) {
    if (p.n_decode > 0) {
        constexpr int MAXLDS = LA_DEC_WAVES * 16 * (WS * 64 + 32) + LA_DEC_WAVES / 2 * 3 * 1024;
        static const int rc = wa_lds(window_decode_kernel<WS, EX>, MAXLDS);
        if (rc != OMNI_OK) return rc;
        const int lds = LA_DEC_WAVES * 16 * (p.vp * 2 + 32) + LA_DEC_WAVES / 2 * 3 * 1024;
        const int wgs = p.kv_heads * ((a.rep + 15) / 16);
        a.nsplit = p.workspace ? la_split_count(wgs * p.n_decode, p.window > 0 && p.window < p.max_keys ? p.window + 15 : p.max_keys) : 1;
        hipLaunchKernelGGL((window_decode_kernel<WS, EX>), dim3(wgs, p.n_decode, a.nsplit), dim3(64 * LA_DEC_WAVES), lds, st, a);
        OMNI_CHECK_LAUNCH("omni_window_attn(decode)");
        if (a.nsplit > 1) {
            hipLaunchKernelGGL(window_merge_kernel, dim3(p.n_decode * p.heads), dim3(64), 0, st, a, a.nsplit);
            OMNI_CHECK_LAUNCH("omni_window_attn(merge)");
        }
    }
    if (p.n_tiles > 0) {
        constexpr int PW = wa_rows_of(WS) / 16, MAXLDS = 2 * LA_KEYS * 2 * (WS * 64 + 32);
        static const int rc = wa_lds(window_prefill_kernel<WS, EX, PW>, MAXLDS);
        if (rc != OMNI_OK) return rc;
        hipLaunchKernelGGL((window_prefill_kernel<WS, EX, PW>), dim3(p.n_tiles, p.kv_heads), dim3(64 * PW), 2 * LA_KEYS * (p.dp * 2 + p.vp * 2 + 64), st, a);
        OMNI_CHECK_LAUNCH("omni_window_attn(prefill)");
    }
    return OMNI_OK;
}

extern "C" int omni_window_attn_run(const omni_window_attn* pp, void* stream) {
    OMNI_CHECK_ARG(pp && pp->q && pp->kc && pp->vc && pp->out && pp->block_table && pp->row_of_tok && pp->positions, "omni_window_attn: null pointer");
    const omni_window_attn& p = *pp;
    OMNI_CHECK_ARG(p.heads > 0 && p.kv_heads > 0 && p.heads % p.kv_heads == 0 && p.kv_heads <= 65535, "omni_window_attn: %d heads over %d key / value heads", p.heads, p.kv_heads);
    OMNI_CHECK_ARG(p.dp > 0 && p.dp % 32 == 0 && p.dp <= WA_PLAIN_MAX && p.vp > 0 && p.vp % 32 == 0 && p.vp <= WA_PLAIN_MAX, "omni_window_attn: dp=%d vp=%d (multiples of 32, <= %d)", p.dp, p.vp, WA_PLAIN_MAX);
    OMNI_CHECK_ARG(p.block_size > 0 && (p.block_size & (p.block_size - 1)) == 0 && p.bt_stride > 0, "omni_window_attn: block_size=%d (a power of two)", p.block_size);
    OMNI_CHECK_ARG(p.n_decode >= 0 && p.n_decode <= p.T && p.n_decode <= 65535 && p.n_tiles >= 0 && (p.n_tiles == 0 || p.tiles) && (p.n_decode == p.T || p.n_tiles > 0 || p.elem == 1),
                   "omni_window_attn: T=%d n_decode=%d n_tiles=%d", p.T, p.n_decode, p.n_tiles);
    OMNI_CHECK_ARG(p.n_tiles == 0 || p.tile_rows == omni_window_attn_tile_rows(p.dp, p.vp), "omni_window_attn: tile_rows=%d (omni_window_attn_tile_rows(%d, %d) = %d)", p.tile_rows, p.dp, p.vp,
                   omni_window_attn_tile_rows(p.dp, p.vp));
    OMNI_CHECK_ARG((p.elem == 0 || (p.elem == 1 && !p.frag)) && p.window >= 0, "omni_window_attn: elem=%d frag=%d window=%d", p.elem, p.frag, p.window);
    OMNI_CHECK_ARG(!p.workspace || p.workspace_bytes >= omni_window_attn_workspace_bytes(p.n_decode, p.heads, p.vp), "omni_window_attn: workspace of %lld bytes", (long long)p.workspace_bytes);
    if (p.T <= 0) return OMNI_OK;
    hipStream_t st = (hipStream_t)stream;
    const int window = p.window > 0 ? p.window : 0x7fffffff, bound = wa_bound(p.dp, p.vp);
    if (p.elem == 1 || !bound) {
        const dim3 grid((unsigned)((int64_t)p.T * p.heads)), block(64);
        if (p.elem == 1) hipLaunchKernelGGL(window_plain_kernel<float>, grid, block, 0, st, p, window);
        else hipLaunchKernelGGL(window_plain_kernel<uint16_t>, grid, block, 0, st, p, window);
        OMNI_CHECK_LAUNCH("omni_window_attn(plain)");
        return OMNI_OK;
    }
    WinArgs a{};
    a.q = (const uint16_t*)p.q; a.kc = (const uint16_t*)p.kc; a.vc = (const uint16_t*)p.vc; a.gate = (const uint16_t*)p.gate; a.sink = p.sink;
    a.out = (uint16_t*)p.out; a.frag = p.frag;
    a.block_table = p.block_table; a.bt_stride = p.bt_stride; a.bs_shift = __builtin_ctz((unsigned)p.block_size); a.bs_mask = p.block_size - 1;
    a.row_of_tok = p.row_of_tok; a.positions = p.positions; a.tiles = p.tiles;
    a.heads = p.heads; a.kv_heads = p.kv_heads; a.rep = p.heads / p.kv_heads; a.ds = p.dp / 32; a.vs = p.vp / 32;
    a.qs = p.scale * LA_LOG2E; a.window = window; a.partial = p.workspace; a.nsplit = 1;
    const bool ex = a.ds == bound && a.vs == bound;
    if (bound == 2) return ex ? wa_run<2, true>(p, a, st) : wa_run<2, false>(p, a, st);
    if (bound == 4) return ex ? wa_run<4, true>(p, a, st) : wa_run<4, false>(p, a, st);
    return ex ? wa_run<8, true>(p, a, st) : wa_run<8, false>(p, a, st);
}
