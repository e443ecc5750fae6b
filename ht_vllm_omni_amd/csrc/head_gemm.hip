// Per-head products of the latent attention (q -> latent space, latent -> values) and the fp32 GEMM of the 32-bit mode.
//
// omni_head_gemm: out[t, h, :] = x[t, h, :] . w[h]^T with K = a head's width (64 .. 576): one wave owns one 16-column tile of one head for up
// to 64 tokens; operands go straight from HBM / L2 into MFMA registers (w fragment-major: 1 KB runs).  Long K with few tiles
// (latent -> values): the four waves of a workgroup split K and combine through LDS in a fixed order.
#include "common.cuh"
#include "gemm_frag.cuh"
#include "../../include/omni_decoder.h"

#define HG_WAVES 4

template <int MT, bool KSPLIT>
__global__ __launch_bounds__(64 * HG_WAVES) void head_gemm_kernel(const uint16_t* __restrict__ x, const uint16_t* __restrict__ w,
                                                                  uint16_t* __restrict__ out, int T, int heads, int n, int k, int frag) {
    __shared__ f32x4 part[KSPLIT ? HG_WAVES : 1][MT][64];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int c = lane & 15, q = lane >> 4;
    const int h = blockIdx.z, m0 = blockIdx.y * (MT * 16);
    const int nt = KSPLIT ? blockIdx.x : blockIdx.x * HG_WAVES + wave;
    const int ntiles = n >> 4, nsteps = k >> 5;
    if (!KSPLIT && nt >= ntiles) return;               // no barrier below on this path
    const uint16_t* wp = w + ((size_t)h * ntiles + nt) * nsteps * 512 + lane * 8;
    const uint16_t* xp[MT];
    const int ldx = heads * k;
#pragma unroll
    for (int i = 0; i < MT; ++i) xp[i] = x + (size_t)min(m0 + i * 16 + c, T - 1) * ldx + h * k + 8 * q;
    f32x4 acc[MT];
#pragma unroll
    for (int i = 0; i < MT; ++i) acc[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
    const int stride = KSPLIT ? HG_WAVES : 1;
    int s = KSPLIT ? wave : 0;
    constexpr int P = 4;                               // k-steps in flight
    for (; s + (P - 1) * stride < nsteps; s += P * stride) {
        u32x4 W[P], X[P][MT];
#pragma unroll
        for (int d = 0; d < P; ++d) {
            W[d] = ld16(wp + (size_t)(s + d * stride) * 512);
#pragma unroll
            for (int i = 0; i < MT; ++i) X[d][i] = ld16(xp[i] + (s + d * stride) * 32);
        }
#pragma unroll
        for (int d = 0; d < P; ++d)
#pragma unroll
            for (int i = 0; i < MT; ++i) acc[i] = mfma16(W[d], X[d][i], acc[i]);
    }
    for (; s < nsteps; s += stride) {
        const u32x4 W = ld16(wp + (size_t)s * 512);
#pragma unroll
        for (int i = 0; i < MT; ++i) acc[i] = mfma16(W, ld16(xp[i] + s * 32), acc[i]);
    }
    auto store = [&](int i, f32x4 v) {                 // lane: token m0 + 16 i + c, columns 16 nt + 4 q ..
        const int m = m0 + i * 16 + c, col = h * n + nt * 16 + 4 * q;
        if (m >= T) return;
        uint16_t* d = out + (frag ? frag_off(m, col, heads * n) : (size_t)m * heads * n + col);
        *reinterpret_cast<uint2*>(d) = make_uint2(pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3]));
    };
    if (!KSPLIT) {
#pragma unroll
        for (int i = 0; i < MT; ++i) store(i, acc[i]);
    } else {
#pragma unroll
        for (int i = 0; i < MT; ++i) part[wave][i][lane] = acc[i];
        __syncthreads();
        for (int i = wave; i < MT; i += HG_WAVES) {
            f32x4 v = part[0][i][lane];
#pragma unroll
            for (int u = 1; u < HG_WAVES; ++u) v += part[u][i][lane];
            store(i, v);
        }
    }
}

extern "C" int omni_head_gemm(const void* x, const void* w, void* out, int T, int heads, int n, int k, int frag, void* stream) {
    OMNI_CHECK_ARG(x && w && out, "omni_head_gemm: null pointer");
    OMNI_CHECK_ARG(heads > 0 && heads <= 65535 && n > 0 && n % 16 == 0 && k > 0 && k % 32 == 0, "omni_head_gemm: heads=%d n=%d (%% 16) k=%d (%% 32)", heads, n, k);
    OMNI_CHECK_ARG(!frag || heads * n % 32 == 0, "omni_head_gemm: fragment-major output needs heads * n %% 32 == 0");
    if (T <= 0) return OMNI_OK;
    const int mt = T > 32 ? 4 : (T > 16 ? 2 : 1);
    const bool ks = k >= 256;
    const dim3 grid(ks ? n / 16 : (n / 16 + HG_WAVES - 1) / HG_WAVES, (T + 16 * mt - 1) / (16 * mt), heads), block(64 * HG_WAVES);
    OMNI_CHECK_ARG(grid.y <= 65535, "omni_head_gemm: T=%d", T);
#define HG(MT_, KS_) hipLaunchKernelGGL((head_gemm_kernel<MT_, KS_>), grid, block, 0, (hipStream_t)stream, (const uint16_t*)x, (const uint16_t*)w, (uint16_t*)out, T, heads, n, k, frag)
    if (ks) { if (mt == 4) HG(4, true); else if (mt == 2) HG(2, true); else HG(1, true); }
    else { if (mt == 4) HG(4, false); else if (mt == 2) HG(2, false); else HG(1, false); }
#undef HG
    OMNI_CHECK_LAUNCH("omni_head_gemm");
    return OMNI_OK;
}

// ---- fp32: 64 x 64 output tile, 16-deep slices of both operands in LDS, 4 x 4 values per thread
#define GF_T 64
#define GF_K 16
__global__ __launch_bounds__(256) void gemm_f32_kernel(const float* __restrict__ x, int ldx, int64_t xb, const float* __restrict__ w, int64_t wb,
                                                       float* __restrict__ out, int ldo, int64_t ob, int M, int N, int K, int act, float ap, float an, const omni_row_table rt) {
    __shared__ float sx[GF_K][GF_T + 4], sw[GF_K][GF_T + 4];
    const int m0 = blockIdx.y * GF_T, n0 = blockIdx.x * GF_T;
    x += blockIdx.z * xb;
    w += blockIdx.z * wb;
    out += blockIdx.z * ob;
    const int tx = threadIdx.x & 15, ty = threadIdx.x >> 4;
    const int lr = threadIdx.x >> 2, lk = (threadIdx.x & 3) * 4;      // loader: row of the tile, 4 consecutive k
    float acc[4][4] = {};
    for (int k0 = 0; k0 < K; k0 += GF_K) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int k = k0 + lk + e;
            sx[lk + e][lr] = (m0 + lr < M && k < K) ? x[(size_t)(m0 + lr) * ldx + k] : 0.f;
            sw[lk + e][lr] = (n0 + lr < N && k < K) ? w[(size_t)(n0 + lr) * K + k] : 0.f;
        }
        __syncthreads();
#pragma unroll
        for (int k = 0; k < GF_K; ++k) {
            float a[4], b[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) { a[e] = sx[k][ty * 4 + e]; b[e] = sw[k][tx * 4 + e]; }
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(a[i], b[j], acc[i][j]);
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int m = m0 + ty * 4 + i;
        if (m >= M) continue;
        const int id = act == OMNI_ACT_GELU_MUL ? rt.ids[m] : -1;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int n = n0 + tx * 4 + j;
            if (n >= N) continue;
            float v = acc[i][j];
            if (act == OMNI_ACT_XIELU) v = xielu(v, ap, an);
            else if (act == OMNI_ACT_RELU2) v = relu2(v);
            else if (act == OMNI_ACT_GELU_MUL) v = id >= 0 && id < rt.rows ? gelu_tanh(v) * reinterpret_cast<const float*>(rt.table)[(size_t)id * rt.ld + n] : 0.f;
            out[(size_t)m * ldo + n] = v;
        }
    }
}

extern "C" int omni_gemm_f32(const float* x, int ldx, int64_t xb, const float* w, int64_t wb, float* out, int ldo, int64_t ob, int M, int N, int K,
                             int batch, int act, float act_p, float act_n, void* stream) {
    OMNI_CHECK_ARG(x && w && out, "omni_gemm_f32: null pointer");
    OMNI_CHECK_ARG(N > 0 && K > 0 && ldx >= K && ldo >= N && batch >= 1 && batch <= 65535 && act >= OMNI_ACT_NONE && act <= OMNI_ACT_RELU2, "omni_gemm_f32: N=%d K=%d ldx=%d ldo=%d batch=%d act=%d", N, K, ldx, ldo, batch, act);
    if (M <= 0) return OMNI_OK;
    const dim3 grid((N + GF_T - 1) / GF_T, (M + GF_T - 1) / GF_T, batch);
    OMNI_CHECK_ARG(grid.y <= 65535, "omni_gemm_f32: M=%d", M);
    hipLaunchKernelGGL(gemm_f32_kernel, grid, dim3(256), 0, (hipStream_t)stream, x, ldx, xb, w, wb, out, ldo, ob, M, N, K, act, act_p, act_n, omni_row_table{});
    OMNI_CHECK_LAUNCH("omni_gemm_f32");
    return OMNI_OK;
}

extern "C" int omni_gemm_f32_rows(const float* x, int ldx, const float* w, float* out, int ldo, int M, int N, int K, const omni_row_table* rt, void* stream) {
    OMNI_CHECK_ARG(x && w && out && rt && rt->table && rt->ids, "omni_gemm_f32_rows: null pointer");
    OMNI_CHECK_ARG(N > 0 && K > 0 && ldx >= K && ldo >= N && rt->rows > 0 && rt->ld >= N, "omni_gemm_f32_rows: N=%d K=%d ldx=%d ldo=%d, table of %d rows, ld %d", N, K, ldx, ldo, rt->rows, rt->ld);
    if (M <= 0) return OMNI_OK;
    const dim3 grid((N + GF_T - 1) / GF_T, (M + GF_T - 1) / GF_T, 1);
    OMNI_CHECK_ARG(grid.y <= 65535, "omni_gemm_f32_rows: M=%d", M);
    hipLaunchKernelGGL(gemm_f32_kernel, grid, dim3(256), 0, (hipStream_t)stream, x, ldx, (int64_t)0, w, (int64_t)0, out, ldo, (int64_t)0, M, N, K, OMNI_ACT_GELU_MUL, 0.f, 0.f, *rt);
    OMNI_CHECK_LAUNCH("omni_gemm_f32_rows");
    return OMNI_OK;
}
