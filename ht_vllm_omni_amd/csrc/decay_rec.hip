// Linear recurrence with one decay per head (include/omni_decoder.h omni_decay_rec): S <- decay S + k v^T, out = S^T q, fp32 state per sequence.
//
//   rec_run_kernel          token by token: a workgroup keeps 64 or 128 columns of one head's S in registers while it walks its tokens.  A decoded token
//                           is a run of one: S is read and written once -- that traffic is the op's bound
//   chunks of 128 tokens, for prompts (matrix cores; a decay's powers enter as fp32 factors, fp32 operands as three bf16 terms whose sum is the value):
//   rec_chunk_state_kernel  what a chunk adds to S:  sum_j decay^(n-1-j) k_j v_j^T, every chunk on its own
//   rec_scan_kernel         S at every chunk's start, in place of its contribution, and the sequence's new state
//   rec_chunk_out_kernel    out_i = decay^(i+1) S_start^T q_i + sum_(j <= i) decay^(i-j) (q_i . k_j) v_j
#include "attn_tile.cuh"
#include "row_io.cuh"

#define RC_T OMNI_REC_CHUNK
#define RC_VB 128                // value columns of an output workgroup
#define RC_VPITCH (RC_VB * 2 + 32)

__device__ __forceinline__ float rc_silu(float z) { return z * sigmoidf_(z); }

// ---- token by token.  Threads: CQ column quads x 256 / CQ row groups; row group g owns rows g, g + 256 / CQ, ...
// RAW: projections fp32 (partial sums), SiLU here; else bf16 behind it
template <int CQ, int MAXR, bool RAW>
__global__ __launch_bounds__(256) void rec_run_kernel(const omni_decay_rec a, const int32_t* items) {
    constexpr int RG = 256 / CQ;
    extern __shared__ __attribute__((aligned(16))) float qk_lds[];     // q | k of the token
    __shared__ f32x4 red[4][CQ];
    const int tid = threadIdx.x, h = blockIdx.y, item = blockIdx.z;
    const int t0 = items ? items[2 * item] : item, n = items ? items[2 * item + 1] : 1;
    const int row = a.row_of_tok[t0];
    if (a.num_live && row >= *a.num_live) return;
    const int cq = tid % CQ, g = tid / CQ, col = (blockIdx.x * CQ + cq) * 4;
    const bool mine = col < a.vp;
    float* sq = qk_lds;
    float* sk = qk_lds + a.dp;
    float* st = a.state + ((size_t)a.state_slot[row] * a.heads + h) * a.dp * a.vp + col;
    const bool zero = a.positions[t0] == 0;
    f32x4 S[MAXR];
#pragma unroll
    for (int i = 0; i < MAXR; ++i) {
        S[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
        const int d = g + RG * i;
        if (mine && !zero && d < a.dp) S[i] = *reinterpret_cast<const f32x4*>(st + (size_t)d * a.vp);
    }
    const float decay = a.decay[h];
    auto value = [&](int t, int c, float (&v)[4]) {
        if constexpr (RAW) {
            ld4_slabs(reinterpret_cast<const float*>(a.proj) + (size_t)t * a.ld + c, a.slabs, a.slab_stride, v);
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = rc_silu(v[e]);
        } else {
            ld4<uint16_t>(reinterpret_cast<const uint16_t*>(a.proj) + (size_t)t * a.ld + c, v);
        }
    };
    const int kcol = a.heads * a.dp, vcol = 2 * a.heads * a.dp;
    for (int t = t0; t < t0 + n; ++t) {
        for (int c = tid * 4; c < 2 * a.dp; c += 1024) {
            float z[4];
            value(t, c < a.dp ? h * a.dp + c : kcol + h * a.dp + c - a.dp, z);
            st4<float>(qk_lds + c, z);
        }
        float v[4] = {0.f, 0.f, 0.f, 0.f};
        if (mine) value(t, vcol + h * a.vp + col, v);
        __syncthreads();                              // q and k of this token
        f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < MAXR; ++i) {
            const int d = g + RG * i;
            if (d >= a.dp) continue;
            const float qd = sq[d], kd = sk[d];
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                S[i][e] = fmaf(decay, S[i][e], kd * v[e]);
                o[e] = fmaf(qd, S[i][e], o[e]);
            }
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = xor32_sum(CQ == 16 ? xor16_sum(o[e]) : o[e]);
        if ((tid & 63) < CQ) red[tid >> 6][cq] = o;
        __syncthreads();                              // the waves' sums (and: nobody reads this token's q, k any more)
        if (tid < CQ && mine) {
            const f32x4 s = (red[0][cq] + red[1][cq]) + (red[2][cq] + red[3][cq]);
            *reinterpret_cast<f32x4*>(a.out + ((size_t)t * a.heads + h) * a.vp + col) = s;
        }
    }
    if (!mine) return;
#pragma unroll
    for (int i = 0; i < MAXR; ++i) {
        const int d = g + RG * i;
        if (d < a.dp) *reinterpret_cast<f32x4*>(st + (size_t)d * a.vp) = S[i];
    }
}

// ---- chunks
// tokens [t0, t0 + n) of a [tokens, ld] bf16 array, up to P 32-wide pieces from column c0, through registers -> row-major LDS image of RC_T rows; rows
// past n are zero
template <int THREADS, int P>
struct RcTile {
    static constexpr int R = RC_T * 4 / THREADS;
    u32x4 v[R][P];
    __device__ __forceinline__ void load(const uint16_t* src, int ld, int t0, int n, int c0, int pieces) {
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const int tok = (threadIdx.x >> 2) + r * (THREADS / 4);
            const uint16_t* p = src + (size_t)(t0 + min(tok, n - 1)) * ld + c0 + 8 * (threadIdx.x & 3);
#pragma unroll
            for (int s = 0; s < P; ++s)
                if (s < pieces) v[r][s] = ld16(p + 32 * s);
        }
    }
    __device__ __forceinline__ void store(unsigned char* img, int pitch, int n, int pieces) const {
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const int tok = (threadIdx.x >> 2) + r * (THREADS / 4);
#pragma unroll
            for (int s = 0; s < P; ++s)
                if (s < pieces) *reinterpret_cast<u32x4*>(img + tok * pitch + (32 * s + 8 * (threadIdx.x & 3)) * 2) = tok < n ? v[r][s] : (u32x4){0, 0, 0, 0};
        }
    }
};

// D[v][d] = V^T . K': A = V^T (lane: v, 8 tokens), B = K' (lane: d, the same tokens) = decay^(n-1-j) k_j in three terms
__global__ __launch_bounds__(256, 2) void rec_chunk_state_kernel(const omni_decay_rec a) {
    extern __shared__ __attribute__((aligned(16))) unsigned char img[];
    const int chunk = blockIdx.x, h = blockIdx.y;
    const int t0 = a.chunks[4 * chunk], n = a.chunks[4 * chunk + 1];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c = lane & 15, qk = lane >> 4;
    const int kp = a.dp * 2 + 32, vpitch = a.vp * 2 + 32;
    unsigned char* kimg = img;
    unsigned char* vimg = img + RC_T * kp;
    const uint16_t* src = reinterpret_cast<const uint16_t*>(a.proj);
    constexpr int P = 4;                              // pieces in flight
    for (int s = 0; s < a.dp / 32 || s < a.vp / 32; s += P) {
        RcTile<256, P> k, v;
        k.load(src, a.ld, t0, n, (a.heads + h) * a.dp + 32 * s, a.dp / 32 - s);
        v.load(src, a.ld, t0, n, 2 * a.heads * a.dp + h * a.vp + 32 * s, a.vp / 32 - s);
        k.store(kimg + 64 * s, kp, n, a.dp / 32 - s);
        v.store(vimg + 64 * s, vpitch, n, a.vp / 32 - s);
    }
    const float l2 = a.log2_decay[h];
    float f[RC_T / 32][8];
#pragma unroll
    for (int ks = 0; ks < RC_T / 32; ++ks)
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const int back = n - 1 - (32 * ks + la_slot(qk, j));
            f[ks][j] = back >= 0 ? exp2_w(l2 * (float)back) : 0.f;
        }
    __syncthreads();
    float* out = a.chunk_states + ((size_t)chunk * a.heads + h) * a.dp * a.vp;
    const int dt_n = a.dp >> 4, vt_n = a.vp >> 4, steps = (n + 31) >> 5;
    for (int dt = wave; dt < dt_n; dt += 4) {
        u32x4 B[RC_T / 32][3];
#pragma unroll
        for (int ks = 0; ks < RC_T / 32; ++ks) {
            const u32x4 k = la_transposed_at(kimg + 32 * ks * kp, kp, dt, c, qk);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                uint32_t hi, mid, lo;
                split3(bf_lo(k[e]) * f[ks][2 * e], bf_hi(k[e]) * f[ks][2 * e + 1], hi, mid, lo);
                B[ks][0][e] = hi; B[ks][1][e] = mid; B[ks][2][e] = lo;
            }
        }
        for (int v0 = 0; v0 < vt_n; v0 += 2) {        // (vt_n is even)
            f32x4 acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
            for (int ks = 0; ks < RC_T / 32; ++ks) {
                if (ks >= steps) break;
                u32x4 A[2];
#pragma unroll
                for (int v = 0; v < 2; ++v) A[v] = la_transposed_at(vimg + 32 * ks * vpitch, vpitch, v0 + v, c, qk);
#pragma unroll
                for (int i = 2; i >= 0; --i)
#pragma unroll
                    for (int v = 0; v < 2; ++v) acc[v] = mfma16(A[v], B[ks][i], acc[v]);
            }
#pragma unroll
            for (int v = 0; v < 2; ++v) *reinterpret_cast<f32x4*>(out + (size_t)(16 * dt + c) * a.vp + 16 * (v0 + v) + 4 * qk) = acc[v];
        }
    }
}

// four state values per thread, the sequence's chunks in order
__global__ __launch_bounds__(256) void rec_scan_kernel(const omni_decay_rec a) {
    const int h = blockIdx.y, c0 = a.segs[2 * blockIdx.z], nc = a.segs[2 * blockIdx.z + 1];
    const int e = (blockIdx.x * 256 + threadIdx.x) * 4, size = a.dp * a.vp;
    if (e >= size) return;
    const int t0 = a.chunks[4 * c0], row = a.row_of_tok[t0];
    if (a.num_live && row >= *a.num_live) return;
    const float l2 = a.log2_decay[h];
    float* st = a.state + ((size_t)a.state_slot[row] * a.heads + h) * size + e;
    float* cs = a.chunk_states + ((size_t)c0 * a.heads + h) * size + e;
    const size_t stride = (size_t)a.heads * size;
    f32x4 S = {0.f, 0.f, 0.f, 0.f};
    if (a.positions[t0] != 0) S = *reinterpret_cast<const f32x4*>(st);
    constexpr int P = 4;
    f32x4 x[P];
    for (int i = 0; i < nc; i += P) {
#pragma unroll
        for (int p = 0; p < P; ++p)
            if (i + p < nc) x[p] = *reinterpret_cast<const f32x4*>(cs + (i + p) * stride);
#pragma unroll
        for (int p = 0; p < P; ++p) {
            if (i + p >= nc) continue;
            const float f = exp2_w(l2 * (float)a.chunks[4 * (c0 + i + p) + 1]);
            *reinterpret_cast<f32x4*>(cs + (i + p) * stride) = S;
#pragma unroll
            for (int k = 0; k < 4; ++k) S[k] = fmaf(f, S[k], x[p][k]);
        }
    }
    *reinterpret_cast<f32x4*>(st) = S;
}

// one chunk, one head, up to RC_VB value columns: eight waves, 16 tokens each; a lane owns one token (its query row)
template <int DS>
__global__ __launch_bounds__(512, 2) void rec_chunk_out_kernel(const omni_decay_rec a) {
    constexpr int dp = DS * 32, KP = dp * 2 + 32;
    constexpr int PLANE = 32 * RC_VPITCH;
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];      // V image | K image, before it: three planes of 32 state rows
    const int chunk = blockIdx.x, h = blockIdx.y, vb0 = blockIdx.z * RC_VB, vcols = min(RC_VB, a.vp - vb0), nvt = vcols >> 4;
    const int t0 = a.chunks[4 * chunk], n = a.chunks[4 * chunk + 1];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, qk = lane >> 4;
    unsigned char* vimg = lds;
    unsigned char* kimg = lds + RC_T * RC_VPITCH;
    const uint16_t* src = reinterpret_cast<const uint16_t*>(a.proj);
    const int i = wave * 16 + c;
    const uint16_t* qrow = src + (size_t)(t0 + min(i, n - 1)) * a.ld + h * dp;
    const float l2 = a.log2_decay[h];
    const bool carry = a.chunks[4 * chunk + 2] != 0 || a.positions[t0] != 0;      // S_start is not zero
    f32x4 O[RC_VB / 16];
#pragma unroll
    for (int v = 0; v < RC_VB / 16; ++v) O[v] = (f32x4){0.f, 0.f, 0.f, 0.f};
    const float* cs = a.chunk_states + ((size_t)chunk * a.heads + h) * dp * a.vp + vb0;
    const int sr = tid >> 4, sc = (tid & 15) * 8;     // this thread's piece of a 32-row slab of states: 8 columns
    f32x4 x[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
    auto slab = [&](int s) {
        if (sc >= vcols) return;
        const float* p = cs + (size_t)(32 * s + sr) * a.vp + sc;
        x[0] = *reinterpret_cast<const f32x4*>(p);
        x[1] = *reinterpret_cast<const f32x4*>(p + 4);
    };
    // everything the chunk reads is on its way before the first wait, in the order it is needed
    if (carry) slab(0);
    RcTile<512, RC_VB / 32> vt;
    RcTile<512, DS> kt_;
    vt.load(src, a.ld, t0, n, 2 * a.heads * dp + h * a.vp + vb0, vcols / 32);
    kt_.load(src, a.ld, t0, n, (a.heads + h) * dp, DS);
    if (carry) {                                      // (uniform)
#pragma unroll 1
        for (int s = 0; s < DS; ++s) {
            u32x4 w[3];
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                uint32_t hi, mid, lo;
                split3(x[e >> 1][2 * (e & 1)], x[e >> 1][2 * (e & 1) + 1], hi, mid, lo);
                w[0][e] = hi; w[1][e] = mid; w[2][e] = lo;
            }
            if (s) __syncthreads();                   // the slab before has been read
#pragma unroll
            for (int p = 0; p < 3; ++p) *reinterpret_cast<u32x4*>(kimg + p * PLANE + sr * RC_VPITCH + sc * 2) = w[p];
            if (s + 1 < DS) slab(s + 1);
            // the lane's query, dimensions in the order of the contraction slots
            const u32x2 qa = *reinterpret_cast<const u32x2*>(qrow + 32 * s + 4 * qk), qb = *reinterpret_cast<const u32x2*>(qrow + 32 * s + 16 + 4 * qk);
            const u32x4 B = {qa[0], qa[1], qb[0], qb[1]};
            __syncthreads();
#pragma unroll
            for (int v = 0; v < RC_VB / 16; ++v) {
                if (v >= nvt) break;
#pragma unroll
                for (int p = 2; p >= 0; --p) O[v] = mfma16(la_transposed_at(kimg + p * PLANE, RC_VPITCH, v, c, qk), B, O[v]);
            }
        }
        const float f = exp2_w(l2 * (float)(i + 1));
#pragma unroll
        for (int v = 0; v < RC_VB / 16; ++v) O[v] *= f;
        __syncthreads();                              // the planes have been read
    }
    vt.store(vimg, RC_VPITCH, n, vcols / 32);
    kt_.store(kimg, KP, n, DS);
    u32x4 Q[DS];
#pragma unroll
    for (int s = 0; s < DS; ++s) Q[s] = ld16(qrow + 32 * s + 8 * qk);
    __syncthreads();
    if (wave * 16 >= n) return;                       // (no barrier below)
    for (int j0 = 0; j0 <= wave * 16 + 15; j0 += 32) {
        f32x4 S[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
        for (int s = 0; s < DS; ++s)
#pragma unroll
            for (int kt = 0; kt < 2; ++kt)
                S[kt] = mfma16(*reinterpret_cast<const u32x4*>(kimg + (j0 + 16 * kt + c) * KP + (32 * s + 8 * qk) * 2), Q[s], S[kt]);
        u32x4 w[3];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            float p[2];
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                const int j = 2 * e + u, back = i - (j0 + la_slot(qk, j));
                p[u] = back >= 0 ? S[j >> 2][j & 3] * exp2_w(l2 * (float)back) : 0.f;
            }
            uint32_t hi, mid, lo;
            split3(p[0], p[1], hi, mid, lo);
            w[0][e] = hi; w[1][e] = mid; w[2][e] = lo;
        }
#pragma unroll
        for (int v = 0; v < RC_VB / 16; ++v) {
            if (v >= nvt) break;
            const u32x4 A = la_transposed_at(vimg + j0 * RC_VPITCH, RC_VPITCH, v, c, qk);
#pragma unroll
            for (int p = 2; p >= 0; --p) O[v] = mfma16(A, w[p], O[v]);
        }
    }
    if (i >= n) return;
    float* o = a.out + ((size_t)(t0 + i) * a.heads + h) * a.vp + vb0 + 4 * qk;
#pragma unroll
    for (int v = 0; v < RC_VB / 16; ++v)
        if (v < nvt) *reinterpret_cast<f32x4*>(o + 16 * v) = O[v];
}

// ---- host side
template <int CQ, bool RAW>
static void rec_runs_launch(const omni_decay_rec& a, const int32_t* items, int n, hipStream_t st) {
    constexpr int RG = 256 / CQ;
    const dim3 grid((a.vp + 4 * CQ - 1) / (4 * CQ), a.heads, n), block(256);
    const size_t lds = 2 * (size_t)a.dp * sizeof(float);
    if (a.dp <= 4 * RG) hipLaunchKernelGGL((rec_run_kernel<CQ, 4, RAW>), grid, block, lds, st, a, items);
    else if (a.dp <= 8 * RG) hipLaunchKernelGGL((rec_run_kernel<CQ, 8, RAW>), grid, block, lds, st, a, items);
    else if (a.dp <= 16 * RG) hipLaunchKernelGGL((rec_run_kernel<CQ, 16, RAW>), grid, block, lds, st, a, items);
    else hipLaunchKernelGGL((rec_run_kernel<CQ, 32, RAW>), grid, block, lds, st, a, items);
}

template <bool RAW>
static int rec_runs(const omni_decay_rec& a, const int32_t* items, int n, hipStream_t st) {
    if (n <= 0) return OMNI_OK;
    if (a.vp > 64 && a.dp <= 256) rec_runs_launch<32, RAW>(a, items, n, st);
    else rec_runs_launch<16, RAW>(a, items, n, st);
    OMNI_CHECK_LAUNCH("omni_decay_rec(runs)");
    return OMNI_OK;
}

template <int DS>
static int rec_out(const omni_decay_rec& a, hipStream_t st) {
    constexpr int KIMG = RC_T * (DS * 64 + 32), PLANES = 3 * 32 * RC_VPITCH, LDS = RC_T * RC_VPITCH + (KIMG > PLANES ? KIMG : PLANES);
    static const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(rec_chunk_out_kernel<DS>), hipFuncAttributeMaxDynamicSharedMemorySize, LDS);
    if (e != hipSuccess) { omni_set_error("omni_decay_rec: LDS attribute: %s", hipGetErrorString(e)); return OMNI_EHIP; }
    hipLaunchKernelGGL(rec_chunk_out_kernel<DS>, dim3(a.n_chunks, a.heads, (a.vp + RC_VB - 1) / RC_VB), dim3(512), LDS, st, a);
    OMNI_CHECK_LAUNCH("omni_decay_rec(out)");
    return OMNI_OK;
}

extern "C" int omni_decay_rec_run(const omni_decay_rec* p, void* stream) {
    OMNI_CHECK_ARG(p && p->proj && p->decay && p->log2_decay && p->state && p->state_slot && p->row_of_tok && p->positions && p->out, "omni_decay_rec: null pointer");
    const omni_decay_rec& a = *p;
    OMNI_CHECK_ARG(a.heads > 0 && a.heads <= 65535 && a.dp > 0 && a.dp % 32 == 0 && a.dp <= 512 && a.vp > 0 && a.vp % 32 == 0 && a.ld >= a.heads * (2 * a.dp + a.vp) && a.ld % 8 == 0,
                   "omni_decay_rec: heads=%d dp=%d (multiple of 32, <= 512) vp=%d ld=%d", a.heads, a.dp, a.vp, a.ld);
    OMNI_CHECK_ARG(a.slabs >= 0 && a.slabs <= OMNI_STREAM_MAX_SPLITS, "omni_decay_rec: slabs=%d", a.slabs);
    OMNI_CHECK_ARG(a.n_decode >= 0 && a.n_decode <= 65535 && a.n_runs >= 0 && a.n_runs <= 65535 && (a.n_runs == 0 || a.runs), "omni_decay_rec: n_decode=%d n_runs=%d", a.n_decode, a.n_runs);
    OMNI_CHECK_ARG(a.n_chunks >= 0 && (a.n_chunks == 0) == (a.n_segs == 0) && a.n_segs <= 65535, "omni_decay_rec: n_chunks=%d n_segs=%d", a.n_chunks, a.n_segs);
    OMNI_CHECK_ARG(a.n_chunks == 0 || (a.chunks && a.segs && a.chunk_states && a.slabs == 0 && a.dp <= OMNI_REC_MAX_DIM && a.vp <= OMNI_REC_MAX_DIM),
                   "omni_decay_rec: chunks take bf16 rows behind SiLU and heads of up to %d (dp=%d vp=%d)", OMNI_REC_MAX_DIM, a.dp, a.vp);
    hipStream_t st = (hipStream_t)stream;
    for (int part = 0; part < 2; ++part) {
        const int32_t* items = part ? a.runs : nullptr;
        const int n = part ? a.n_runs : a.n_decode;
        const int rc = a.slabs > 0 ? rec_runs<true>(a, items, n, st) : rec_runs<false>(a, items, n, st);
        if (rc != OMNI_OK) return rc;
    }
    if (a.n_chunks == 0) return OMNI_OK;
    static const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(rec_chunk_state_kernel), hipFuncAttributeMaxDynamicSharedMemorySize,
                                                    RC_T * 2 * (OMNI_REC_MAX_DIM * 2 + 32));
    if (e != hipSuccess) { omni_set_error("omni_decay_rec: LDS attribute: %s", hipGetErrorString(e)); return OMNI_EHIP; }
    hipLaunchKernelGGL(rec_chunk_state_kernel, dim3(a.n_chunks, a.heads), dim3(256), RC_T * (a.dp * 2 + a.vp * 2 + 64), st, a);
    OMNI_CHECK_LAUNCH("omni_decay_rec(chunk states)");
    hipLaunchKernelGGL(rec_scan_kernel, dim3((a.dp * a.vp / 4 + 255) / 256, a.heads, a.n_segs), dim3(256), 0, st, a);
    OMNI_CHECK_LAUNCH("omni_decay_rec(scan)");
    switch (a.dp / 32) {
#define X(DS_) case DS_: return rec_out<DS_>(a, st);
        X(1) X(2) X(3) X(4) X(5) X(6) X(7) X(8)
#undef X
        default: return OMNI_EINVAL;
    }
}
