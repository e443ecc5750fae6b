// Weight-streaming GEMM of the language models' decode step: out[M <= 64, N] = x[M, K] . W[N, K]^T, both operands fragment-major
// (common.cuh frag_off), every W byte read once.
//
// A workgroup owns NT 16-column tiles for all rows and 1 / S of K (grid.y = S); its 8 waves take the k-steps round-robin, P steps of W and x in
// flight each, and combine through LDS in a fixed order.  What bounds the op at 64 rows is not only W: every workgroup reads all of
// x for its K range, 64 rows against its 16 NT columns of W, so wide tiles with K split over workgroups move the fewest bytes through L2.  The
// S partial sums leave as fp32 slabs [S][M][N]; the row kernels that consume them (decoder_rows.hip) add them up in slab order.
//   out kinds: fp32 slabs (S >= 1) | bf16 row- or fragment-major | the same through an activation (common.cuh), possibly times a row table
#include "common.cuh"
#include "gemm_frag.cuh"
#include "../../include/omni_decoder.h"

#define GS_WAVES 8
#define GS_THREADS (GS_WAVES * 64)
enum { GS_F32 = 0, GS_BF16 = 1, GS_ACT = 2 };

struct StreamArgs {
    const uint16_t* x; const uint16_t* W; void* out;
    int M, N, nsteps, split_steps, oshuf;
    float ap, an;
    int act;
    omni_row_table rt;
};

// P: k-steps in flight per wave: 2 on a grid that fills the chip (4 measured the same or slower at 1 .. 64 rows).
// grid.z: groups of MT row tiles (more than one on narrow products only)
template <int MT, int NT, int KIND, int P>
__global__ __launch_bounds__(GS_THREADS) void gemm_stream_kernel(const StreamArgs a) {
    extern __shared__ __attribute__((aligned(16))) f32x4 part[];      // [wave][NT * MT][lane]
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int k0 = blockIdx.y * a.split_steps, nk = min(a.split_steps, a.nsteps - k0);
    const int m0 = blockIdx.z * MT;
    const uint16_t* wp[NT];
    const uint16_t* xp[MT];
#pragma unroll
    for (int j = 0; j < NT; ++j) wp[j] = a.W + ((size_t)(blockIdx.x * NT + j) * a.nsteps + k0 + wave) * 512 + lane * 8;
#pragma unroll
    for (int i = 0; i < MT; ++i) xp[i] = a.x + ((size_t)min(m0 + i, ((a.M + 15) >> 4) - 1) * a.nsteps + k0 + wave) * 512 + lane * 8;      // row tiles past M: re-read, discarded
    f32x4 acc[NT][MT];
#pragma unroll
    for (int j = 0; j < NT; ++j)
#pragma unroll
        for (int i = 0; i < MT; ++i) acc[j][i] = (f32x4){0.f, 0.f, 0.f, 0.f};
    const int mine = nk > wave ? (nk - wave + GS_WAVES - 1) / GS_WAVES : 0;
    u32x4 W[P][NT], X[P][MT];
    auto load = [&](int d, int s) {
#pragma unroll
        for (int j = 0; j < NT; ++j) W[d][j] = ld16_nt(wp[j] + (size_t)s * (GS_WAVES * 512));
#pragma unroll
        for (int i = 0; i < MT; ++i) X[d][i] = ld16(xp[i] + (size_t)s * (GS_WAVES * 512));
    };
    auto mul = [&](int d) {
#pragma unroll
        for (int j = 0; j < NT; ++j)
#pragma unroll
            for (int i = 0; i < MT; ++i) acc[j][i] = mfma16(W[d][j], X[d][i], acc[j][i]);
    };
    int s = 0;
    if (mine >= P) {                       // whole groups of P steps: no predicated load, each product waits for its own operands only
#pragma unroll
        for (int d = 0; d < P; ++d) load(d, d);
        for (; s + 2 * P <= mine; s += P) {
#pragma unroll
            for (int d = 0; d < P; ++d) {
                mul(d);
                load(d, s + P + d);
            }
        }
#pragma unroll
        for (int d = 0; d < P; ++d) mul(d);
        s += P;
    }
    if (s < mine) {                        // fewer than P steps left
#pragma unroll
        for (int d = 0; d < P - 1; ++d)
            if (s + d < mine) load(d, s + d);
#pragma unroll
        for (int d = 0; d < P - 1; ++d)
            if (s + d < mine) mul(d);
    }
#pragma unroll
    for (int j = 0; j < NT; ++j)
#pragma unroll
        for (int i = 0; i < MT; ++i) part[(wave * (NT * MT) + j * MT + i) * 64 + lane] = acc[j][i];
    __syncthreads();
    for (int it = threadIdx.x; it < NT * MT * 64; it += GS_THREADS) {
        const int l = it & 63, f = it >> 6, j = f / MT, i = f - j * MT;
        const int m = (m0 + i) * 16 + (l & 15), n = (blockIdx.x * NT + j) * 16 + 4 * (l >> 4);
        if (m >= a.M) continue;
        f32x4 v = part[f * 64 + l];
#pragma unroll
        for (int w = 1; w < GS_WAVES; ++w) v += part[(w * (NT * MT) + f) * 64 + l];
        if (KIND == GS_F32) {
            *reinterpret_cast<f32x4*>(reinterpret_cast<float*>(a.out) + ((size_t)blockIdx.y * a.M + m) * a.N + n) = v;
        } else {
            if (KIND == GS_ACT) {
                if (a.act == OMNI_ACT_XIELU) {
#pragma unroll
                    for (int e = 0; e < 4; ++e) v[e] = xielu(v[e], a.ap, a.an);
                } else if (a.act == OMNI_ACT_RELU2) {
#pragma unroll
                    for (int e = 0; e < 4; ++e) v[e] = relu2(v[e]);
                } else {
                    const int id = a.rt.ids[m];
                    uint2 z = make_uint2(0, 0);
                    if (id >= 0 && id < a.rt.rows) z = *reinterpret_cast<const uint2*>(reinterpret_cast<const uint16_t*>(a.rt.table) + (size_t)id * a.rt.ld + n);
                    v[0] = gelu_tanh(v[0]) * bf_lo(z.x); v[1] = gelu_tanh(v[1]) * bf_hi(z.x);
                    v[2] = gelu_tanh(v[2]) * bf_lo(z.y); v[3] = gelu_tanh(v[3]) * bf_hi(z.y);
                }
            }
            uint16_t* d = reinterpret_cast<uint16_t*>(a.out) + (a.oshuf ? frag_off(m, n, a.N) : (size_t)m * a.N + n);
            *reinterpret_cast<uint2*>(d) = make_uint2(pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3]));
        }
    }
}

// Columns per workgroup and K splits.  A workgroup's registers and LDS leave room for one per CU at 64 rows, so a grid runs in rounds of 256; a
// workgroup's time goes with the operand tiles it reads (NT of W and MT of x per k-step) plus its epilogue, a split also costs its consumer.
// Measured at 64 rows: 9216 x 2048 by 3 (192 workgroups) 12.1 us, by 2 (288: two rounds) 15.0; 2048 x 9216 by 2 in 4 splits (256) 11.4, in 6 13.3.
static void gs_policy(int M, int N, int nsteps, bool slabs, int* nt, int* splits) {
    const int tiles = N / 16, mt = M > 32 ? 4 : (M > 16 ? 2 : 1);
    long best = -1;
    for (int n = 1; n <= 4; ++n) {
        if (tiles % n) continue;
        for (int s = 1; s <= (slabs ? OMNI_STREAM_MAX_SPLITS : 1); ++s) {
            if (s > 1 && nsteps / s < 2 * GS_WAVES) break;
            const long rounds = ((long)tiles / n * s + 255) / 256;
            const long cost = rounds * ((n + mt) * ((nsteps + s - 1) / s) + 4 * n * mt) + 12 * s;
            if (best < 0 || cost < best) { best = cost; *nt = n; *splits = s; }
        }
    }
}

template <int MT, int NT, int KIND, int P>
static int gs_launch(const StreamArgs& a, int splits, hipStream_t st) {
    constexpr int LDS = GS_WAVES * NT * MT * 1024;
    if (LDS > 64 * 1024) {
        static const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(gemm_stream_kernel<MT, NT, KIND, P>), hipFuncAttributeMaxDynamicSharedMemorySize, LDS);
        if (e != hipSuccess) { omni_set_error("omni_gemm_stream: LDS attribute: %s", hipGetErrorString(e)); return OMNI_EHIP; }
    }
    hipLaunchKernelGGL((gemm_stream_kernel<MT, NT, KIND, P>), dim3(a.N / (16 * NT), splits, ((a.M + 15) / 16 + MT - 1) / MT), dim3(GS_THREADS), LDS, st, a);
    OMNI_CHECK_LAUNCH("omni_gemm_stream");
    return OMNI_OK;
}

extern "C" int omni_gemm_stream_splits(int M, int N, int K) {
    int nt, s;
    gs_policy(M, N, K / 32, true, &nt, &s);
    return s;
}

static int gs_run(StreamArgs a, int kind, bool one, hipStream_t st) {
    int nt, splits;
    gs_policy(a.M, a.N, a.nsteps, kind == GS_F32 && !one, &nt, &splits);
    a.split_steps = (a.nsteps + splits - 1) / splits;
    const int mt = a.M > 32 ? 4 : (a.M > 16 ? 2 : 1);
    // a narrow product (a side input's gate): its few workgroups would each pull all of x through one CU, so the rows are dealt out as well
    if (a.N / 16 * splits <= 32) {
        if (kind == GS_F32) return gs_launch<1, 1, GS_F32, 4>(a, splits, st);
        return kind == GS_BF16 ? gs_launch<1, 1, GS_BF16, 4>(a, splits, st) : gs_launch<1, 1, GS_ACT, 4>(a, splits, st);
    }
#define GS(MT_, NT_, K_) if (mt == MT_ && nt == NT_ && kind == K_) return gs_launch<MT_, NT_, K_, 2>(a, splits, st);
#define GS_NT(NT_, K_) GS(1, NT_, K_) GS(2, NT_, K_) GS(4, NT_, K_)
#define GS_ALL(K_) GS_NT(1, K_) GS_NT(2, K_) GS_NT(3, K_) GS_NT(4, K_)
    GS_ALL(GS_F32) GS_ALL(GS_BF16) GS_ALL(GS_ACT)
    omni_set_error("omni_gemm_stream: no tile for M=%d N=%d", a.M, a.N);
    return OMNI_EINVAL;
}

#define GS_CHECK(name)                                                                                                                              \
    OMNI_CHECK_ARG(x && w && out, name ": null pointer");                                                                                           \
    OMNI_CHECK_ARG(M >= 1 && M <= 64 && N > 0 && N % 16 == 0 && K > 0 && K % 32 == 0, name ": M=%d (<= 64) N=%d (%% 16) K=%d (%% 32)", M, N, K);    \
    OMNI_CHECK_ARG(!out_frag || N % 32 == 0, name ": out_frag needs N %% 32 == 0 (N=%d)", N)

extern "C" int omni_gemm_stream(const void* x, const void* w, void* out, int M, int N, int K, int kind, int one, float act_p, float act_n, int out_frag, void* stream) {
    GS_CHECK("omni_gemm_stream");
    OMNI_CHECK_ARG(kind >= 0 && kind <= 3 && (!out_frag || kind != GS_F32), "omni_gemm_stream: kind=%d out_frag=%d", kind, out_frag);
    StreamArgs a{(const uint16_t*)x, (const uint16_t*)w, out, M, N, K / 32, 0, out_frag, act_p, act_n, kind == 3 ? OMNI_ACT_RELU2 : OMNI_ACT_XIELU, {}};
    return gs_run(a, kind == 3 ? (int)GS_ACT : kind, one != 0, (hipStream_t)stream);
}

extern "C" int omni_gemm_stream_rows(const void* x, const void* w, void* out, int M, int N, int K, const omni_row_table* rt, int out_frag, void* stream) {
    GS_CHECK("omni_gemm_stream_rows");
    OMNI_CHECK_ARG(rt && rt->table && rt->ids && rt->rows > 0 && rt->ld >= N && rt->ld % 4 == 0, "omni_gemm_stream_rows: table of %d rows, ld %d", rt ? rt->rows : 0, rt ? rt->ld : 0);
    StreamArgs a{(const uint16_t*)x, (const uint16_t*)w, out, M, N, K / 32, 0, out_frag, 0.f, 0.f, OMNI_ACT_GELU_MUL, *rt};
    return gs_run(a, GS_ACT, true, (hipStream_t)stream);
}
