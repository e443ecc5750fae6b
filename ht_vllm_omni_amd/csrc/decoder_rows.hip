// Row-wise kernels of the decoder-only language models (include/omni_decoder.h): everything between two matrix products of a layer.
// The residual stream is fp32; norms, gates and the token-shift state are fp32; only matrix operands are rounded (once) to bf16.
#include "row_io.cuh"

#define DR_THREADS 256
#define DR_WAVES (DR_THREADS / 64)

// sum over the workgroup, result in every thread; `buf` alternates between calls so that one barrier per sum is enough
struct BlockSum {
    float* lds;      // [2][DR_WAVES]
    int flip;
    __device__ __forceinline__ float operator()(float v) {
        v = wave_sum(v);
        float* b = lds + flip * DR_WAVES;
        flip ^= 1;
        if ((threadIdx.x & 63) == 0) b[threadIdx.x >> 6] = v;
        __syncthreads();
        float t = 0.f;
#pragma unroll
        for (int w = 0; w < DR_WAVES; ++w) t += b[w];
        return t;
    }
};

// A workgroup walks `strip` consecutive tokens so that the token shift finds the previous token's NEW stream row in registers; only the
// strip's first token rebuilds its predecessor (or reads it from the sequence's state, or takes zeros).
template <typename E, int MAXC, bool SHIFT>
__global__ __launch_bounds__(DR_THREADS) void stream_rows_kernel(const omni_stream_rows a, int strip) {
    __shared__ float red[2 * DR_WAVES];
    BlockSum bsum{red, 0};
    const int wp = a.wp;
    const E* table = reinterpret_cast<const E*>(a.table);
    const E* mu = reinterpret_cast<const E*>(a.mu);
    const E* yw = reinterpret_cast<const E*>(a.y_w);
    const E* fw = reinterpret_cast<const E*>(a.final_w);
    E* h_out = reinterpret_cast<E*>(a.h_out);
    auto load_new = [&](int t, float (&v)[MAXC][4]) {      // the stream row of token t behind the sublayer that just ran
        if (a.ids) {
            const int id = a.ids[t];
            const bool ok = id >= 0 && id < a.vocab;
#pragma unroll
            for (int c = 0; c < MAXC; ++c) {
                const int k = (c * DR_THREADS + threadIdx.x) * 4;
                v[c][0] = v[c][1] = v[c][2] = v[c][3] = 0.f;
                if (ok && k < wp) ld4<E>(table + (size_t)id * wp + k, v[c]);
                if (a.table_scale != 0.f) {
#pragma unroll
                    for (int e = 0; e < 4; ++e) v[c][e] *= a.table_scale;
                }
            }
            return;
        }
        float y[MAXC][4], ss = 0.f;
#pragma unroll
        for (int c = 0; c < MAXC; ++c) {
            const int k = (c * DR_THREADS + threadIdx.x) * 4;
            v[c][0] = v[c][1] = v[c][2] = v[c][3] = 0.f;
            y[c][0] = y[c][1] = y[c][2] = y[c][3] = 0.f;
            if (k < wp) {
                ld4<float>(a.x_in + (size_t)t * wp + k, v[c]);
                if (a.y) ld4_slabs(a.y + (size_t)t * wp + k, a.y_slabs, a.y_stride, y[c]);
            }
        }
        if (!a.y) return;
        if (a.post) {                                      // the norm takes the sum, not the sublayer's output
#pragma unroll
            for (int c = 0; c < MAXC; ++c)
#pragma unroll
                for (int e = 0; e < 4; ++e) { y[c][e] = fmaf(a.alpha, v[c][e], y[c][e]); v[c][e] = 0.f; }
        }
#pragma unroll
        for (int c = 0; c < MAXC; ++c) ss += sq4_sum(y[c][0], y[c][1], y[c][2], y[c][3]);
        ss = bsum(ss);
        const float r = (yw ? 1.0f : a.gain) / sqrtf(ss / (float)a.width + a.eps);
#pragma unroll
        for (int c = 0; c < MAXC; ++c) {
            if (yw) {
                const int k = (c * DR_THREADS + threadIdx.x) * 4;
                float w[4] = {0.f, 0.f, 0.f, 0.f};
                if (k < wp) ld4<E>(yw + k, w);
#pragma unroll
                for (int e = 0; e < 4; ++e) y[c][e] *= w[e];
            }
#pragma unroll
            for (int e = 0; e < 4; ++e) v[c][e] = fmaf(y[c][e], r, v[c][e]);
        }
    };
    const int i0 = blockIdx.x * strip, i1 = min(i0 + strip, a.rows);
    float cur[MAXC][4], prev[MAXC][4];
    for (int i = i0; i < i1; ++i) {
        const int t = a.sel ? a.sel[i] : i;
        if (SHIFT) {
            const int row = a.row_of_tok[t];
            const bool first = t == 0 || a.row_of_tok[t - 1] != row;
            if (first) {
                const bool zero = a.positions[t] == 0;
                const float* st = a.state + (size_t)a.state_slot[row] * wp;
#pragma unroll
                for (int c = 0; c < MAXC; ++c) {
                    const int k = (c * DR_THREADS + threadIdx.x) * 4;
                    prev[c][0] = prev[c][1] = prev[c][2] = prev[c][3] = 0.f;
                    if (!zero && k < wp) ld4<float>(st + k, prev[c]);
                }
            } else if (i == i0) {
                load_new(t - 1, prev);
            } else {
#pragma unroll
                for (int c = 0; c < MAXC; ++c)
#pragma unroll
                    for (int e = 0; e < 4; ++e) prev[c][e] = cur[c][e];
            }
        }
        load_new(t, cur);
        float rf = 0.f;
        if (!SHIFT && a.use_final) {
            float ss = 0.f;
#pragma unroll
            for (int c = 0; c < MAXC; ++c) ss += sq4_sum(cur[c][0], cur[c][1], cur[c][2], cur[c][3]);
            rf = (fw ? 1.0f : a.final_gain) / sqrtf(bsum(ss) / (float)a.width + a.eps);
        }
#pragma unroll
        for (int c = 0; c < MAXC; ++c) {
            const int k = (c * DR_THREADS + threadIdx.x) * 4;
            if (k >= wp) continue;
            if (a.x_out) st4<float>(a.x_out + (size_t)t * wp + k, cur[c]);
            if (!h_out) continue;
            float h[4];
            if (SHIFT) {
                float m[4];
                ld4<E>(mu + k, m);
#pragma unroll
                for (int e = 0; e < 4; ++e) h[e] = fmaf(prev[c][e] - cur[c][e], m[e], cur[c][e]);
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e) h[e] = a.use_final ? cur[c][e] * rf : cur[c][e];
                if (a.use_final && fw) {
                    float w[4];
                    ld4<E>(fw + k, w);
#pragma unroll
                    for (int e = 0; e < 4; ++e) h[e] *= w[e];
                }
            }
            st4<E>(h_out + (a.frag ? frag_off(i, k, wp) : (size_t)i * wp + k), h);
        }
    }
}

template <typename E, int MAXC>
static void stream_rows_launch(const omni_stream_rows& a, int strip, hipStream_t st) {
    const dim3 grid((a.rows + strip - 1) / strip), block(DR_THREADS);
    if (a.mu) hipLaunchKernelGGL((stream_rows_kernel<E, MAXC, true>), grid, block, 0, st, a, strip);
    else hipLaunchKernelGGL((stream_rows_kernel<E, MAXC, false>), grid, block, 0, st, a, strip);
}

template <typename E>
static int stream_rows_pick(const omni_stream_rows& a, int strip, hipStream_t st) {
    const int chunks = (a.wp / 4 + DR_THREADS - 1) / DR_THREADS;
    if (chunks <= 1) stream_rows_launch<E, 1>(a, strip, st);
    else if (chunks <= 2) stream_rows_launch<E, 2>(a, strip, st);
    else if (chunks <= 4) stream_rows_launch<E, 4>(a, strip, st);
    else stream_rows_launch<E, 8>(a, strip, st);
    OMNI_CHECK_LAUNCH("omni_stream_rows");
    return OMNI_OK;
}

extern "C" int omni_stream_rows_run(const omni_stream_rows* p, void* stream) {
    OMNI_CHECK_ARG(p && (p->ids ? p->table != nullptr : p->x_in != nullptr) && (p->x_out || p->h_out), "omni_stream_rows: null pointer");
    const omni_stream_rows& a = *p;
    OMNI_CHECK_ARG(a.width > 0 && a.wp >= a.width && a.wp % 32 == 0 && a.wp <= DR_THREADS * 4 * 8, "omni_stream_rows: width=%d wp=%d (multiple of 32, <= 8192)", a.width, a.wp);
    OMNI_CHECK_ARG(a.y_slabs <= OMNI_STREAM_MAX_SPLITS, "omni_stream_rows: y_slabs=%d", a.y_slabs);
    OMNI_CHECK_ARG(a.elem == 0 || a.elem == 1, "omni_stream_rows: elem=%d", a.elem);
    OMNI_CHECK_ARG(!a.frag || a.elem == 0, "omni_stream_rows: fragment-major output is bf16");
    OMNI_CHECK_ARG(!a.mu || (a.state && a.state_slot && a.row_of_tok && a.positions && !a.sel && !a.use_final), "omni_stream_rows: token shift needs state, rows and positions, and no selection");
    OMNI_CHECK_ARG(!a.sel || !a.x_out, "omni_stream_rows: a selection writes h only");
    OMNI_CHECK_ARG(!a.post || (a.y && !a.ids), "omni_stream_rows: the norm behind the sum needs y");
    // (a strip's first token and the shift read rows of x_in that another workgroup may already have rewritten: never in place)
    OMNI_CHECK_ARG(a.x_out == nullptr || a.x_out != a.x_in, "omni_stream_rows: x_out must not be x_in");
    if (a.rows <= 0) return OMNI_OK;
    const int strip = a.mu && a.rows > 1024 ? 4 : 1;
    return a.elem ? stream_rows_pick<float>(a, strip, (hipStream_t)stream) : stream_rows_pick<uint16_t>(a, strip, (hipStream_t)stream);
}

// ---- latents: norms, cache write, gates, token-shift state.  One workgroup per token.
template <typename E>
__global__ __launch_bounds__(DR_THREADS) void latent_write_kernel(const omni_latent_write a) {
    extern __shared__ __attribute__((aligned(16))) float sp[];     // the token's projections, partial sums added up
    __shared__ float red[2][DR_WAVES];
    const int t = blockIdx.x;
    const int row = a.row_of_tok[t], pos = a.positions[t];
    const bool live = !a.num_live || row < *a.num_live;
    const int blk = a.block_table[(size_t)row * a.bt_stride + pos / a.block_size];
    const bool last = a.state && (t == a.T - 1 || a.row_of_tok[t + 1] != row);
    const int slot = a.state ? a.state_slot[row] : 0;
    const float* y = a.proj + (size_t)t * a.ld;
    float sq = 0.f, sk = 0.f;
    for (int k = threadIdx.x * 4; k < a.ld; k += DR_THREADS * 4) {
        float v[4];
        ld4_slabs(y + k, a.slabs, a.slab_stride, v);
        st4<float>(sp + k, v);
        const float ss = sq4_sum(v[0], v[1], v[2], v[3]);          // (padded columns hold zeros; qp and rp are multiples of 4)
        if (k < a.qp) sq += ss;
        else if (k < a.qp + a.rp) sk += ss;
    }
    sq = wave_sum(sq);
    sk = wave_sum(sk);
    if ((threadIdx.x & 63) == 0) { red[0][threadIdx.x >> 6] = sq; red[1][threadIdx.x >> 6] = sk; }
    __syncthreads();
    sq = sk = 0.f;
#pragma unroll
    for (int w = 0; w < DR_WAVES; ++w) { sq += red[0][w]; sk += red[1][w]; }
    const float rq = 1.0f / sqrtf(sq / (float)a.q_rank + a.eps), rk = 1.0f / sqrtf(sk / (float)a.kv_rank + a.eps);
    E* cq = reinterpret_cast<E*>(a.cq);
    const E* qw = reinterpret_cast<const E*>(a.qw);
    for (int k = threadIdx.x * 4; k < a.qp; k += DR_THREADS * 4) {
        float v[4], w[4];
        ld4<float>(sp + k, v);
        ld4<E>(qw + k, w);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = v[e] * rq * w[e];
        st4<E>(cq + (a.frag ? frag_off(t, k, a.qp) : (size_t)t * a.qp + k), v);
    }
    if (a.gate)
        for (int h = threadIdx.x; h < a.heads; h += DR_THREADS) a.gate[(size_t)t * a.heads + h] = 1.0f / (1.0f + expf(-sp[a.qp + a.rp + h]));
    if (!live) return;
    E* dst = reinterpret_cast<E*>(a.cache) + ((size_t)blk * a.block_size + pos % a.block_size) * a.rp;
    const E* kw = reinterpret_cast<const E*>(a.kw);
    for (int k = threadIdx.x * 4; k < a.rp; k += DR_THREADS * 4) {
        float v[4], w[4];
        ld4<float>(sp + a.qp + k, v);
        ld4<E>(kw + k, w);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = v[e] * rk * w[e];
        st4<E>(dst + k, v);
    }
    if (last)
        for (int k = threadIdx.x * 4; k < a.wp; k += DR_THREADS * 4) {
            float v[4];
            ld4<float>(a.x + (size_t)t * a.wp + k, v);
            st4<float>(a.state + (size_t)slot * a.wp + k, v);
        }
}

extern "C" int omni_latent_write_run(const omni_latent_write* p, void* stream) {
    OMNI_CHECK_ARG(p && p->proj && p->qw && p->kw && p->cq && p->cache && p->block_table && p->row_of_tok && p->positions, "omni_latent_write: null pointer");
    const omni_latent_write& a = *p;
    OMNI_CHECK_ARG(a.q_rank > 0 && a.kv_rank > 0 && a.qp >= a.q_rank && a.rp >= a.kv_rank && a.qp % 32 == 0 && a.rp % 32 == 0 && a.ld % 4 == 0 &&
                   a.ld >= a.qp + a.rp + (a.gate ? a.heads : 0), "omni_latent_write: q %d / %d, kv %d / %d, ld %d", a.q_rank, a.qp, a.kv_rank, a.rp, a.ld);
    OMNI_CHECK_ARG(a.block_size > 0 && a.bt_stride > 0 && a.heads > 0, "omni_latent_write: block_size=%d bt_stride=%d", a.block_size, a.bt_stride);
    OMNI_CHECK_ARG(!a.state || (a.x && a.state_slot && a.wp % 4 == 0), "omni_latent_write: state needs the stream rows and slots");
    OMNI_CHECK_ARG(a.elem == 1 || a.elem == 0, "omni_latent_write: elem=%d", a.elem);
    OMNI_CHECK_ARG(!a.frag || a.elem == 0, "omni_latent_write: fragment-major output is bf16");
    OMNI_CHECK_ARG(a.slabs <= OMNI_STREAM_MAX_SPLITS, "omni_latent_write: slabs=%d", a.slabs);
    OMNI_CHECK_ARG(a.ld <= 15 * 1024, "omni_latent_write: ld=%d (<= 15360: a token's projections are staged in LDS)", a.ld);
    if (a.T <= 0) return OMNI_OK;
    const size_t lds = (size_t)a.ld * sizeof(float);
    if (a.elem) hipLaunchKernelGGL(latent_write_kernel<float>, dim3(a.T), dim3(DR_THREADS), lds, (hipStream_t)stream, a);
    else hipLaunchKernelGGL(latent_write_kernel<uint16_t>, dim3(a.T), dim3(DR_THREADS), lds, (hipStream_t)stream, a);
    OMNI_CHECK_LAUNCH("omni_latent_write");
    return OMNI_OK;
}

// ---- grouped attention: norms over whole projections, rotation, cache write, gate.  Three workgroups per token, by what they read: queries | keys and
// values | gate.  Queries and keys stay in LDS between the norm's sum and the rotation (a pair's other half belongs to another thread)
template <typename E, bool WIDE>                       // WIDE: half a rotation is a multiple of 4, so 4 consecutive dimensions have 4 consecutive partners
__global__ __launch_bounds__(DR_THREADS) void qkv_write_kernel(const omni_qkv_write a) {
    extern __shared__ __attribute__((aligned(16))) float sp[];     // q or k of the token, partial sums added up
    __shared__ float red[DR_WAVES];
    const int t = blockIdx.x, part = blockIdx.y;
    const int nq = a.heads * a.dp, nk = a.kc ? a.kv_heads * a.dp : 0, nv = a.kc ? a.kv_heads * a.vp : 0, ng = a.heads * a.vp;
    const float* y = a.proj + (size_t)t * a.ld;
    if (part == 2) {
        for (int k = threadIdx.x * 4; k < ng; k += DR_THREADS * 4) {
            float v[4];
            ld4_slabs(y + nq + nk + nv + k, a.slabs, a.slab_stride, v);
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = sigmoidf_(v[e]);
            st4<E>(reinterpret_cast<E*>(a.gate) + (size_t)t * ng + k, v);
        }
        return;
    }
    const int row = a.row_of_tok[t], pos = a.positions[t];
    if (part == 1 && (!a.kc || (a.num_live && row >= *a.num_live))) return;
    // cache rows of this token: head g at base + g * block_size
    const size_t base = part ? (size_t)a.block_table[(size_t)row * a.bt_stride + pos / a.block_size] * a.kv_heads * a.block_size + pos % a.block_size : 0;
    const int n = part ? nk : nq, heads = part ? a.kv_heads : a.heads;
    const E* w = reinterpret_cast<const E*>(part ? a.kw : a.qw);
    if (part) y += nq;
    float ss = 0.f;
    for (int k = threadIdx.x * 4; k < n; k += DR_THREADS * 4) {
        float v[4];
        ld4_slabs(y + k, a.slabs, a.slab_stride, v);
        st4<float>(sp + k, v);
        ss += sq4_sum(v[0], v[1], v[2], v[3]);
    }
    if (part)
        for (int k = threadIdx.x * 4; k < nv; k += DR_THREADS * 4) {
            float v[4];
            ld4_slabs(y + nk + k, a.slabs, a.slab_stride, v);
            const int g = k / a.vp, d = k - g * a.vp;
            st4<E>(reinterpret_cast<E*>(a.vc) + (base + (size_t)g * a.block_size) * a.vp + d, v);
        }
    ss = wave_sum(ss);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int i = 0; i < DR_WAVES; ++i) ss += red[i];
    const float r = w ? 1.0f / sqrtf(ss / (float)(heads * a.dim) + a.eps) : 1.0f;
    const int half = a.rot_dims >> 1;
    const float* cs = a.rot + (size_t)min(pos, a.rot_rows - 1) * a.rot_dims;
    for (int k = threadIdx.x * 4; k < n; k += DR_THREADS * 4) {
        const int hd = k / a.dp, d0 = k - hd * a.dp;
        float v[4], o[4] = {0.f, 0.f, 0.f, 0.f}, wv[4] = {1.f, 1.f, 1.f, 1.f};
        ld4<float>(sp + k, v);
        if (w) ld4<E>(w + k, wv);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = v[e] * r * wv[e];
        if (d0 < a.rot_dims) {                         // (the vector may end past the rotated dimensions)
            float c[4] = {1.f, 1.f, 1.f, 1.f}, sn[4] = {0.f, 0.f, 0.f, 0.f};
            if constexpr (WIDE) {
                const bool lo = d0 < half;
                const int q = lo ? k + half : k - half;
                const float* p = cs + 2 * (lo ? d0 : d0 - half);
                ld4<float>(sp + q, o);
                float wo[4] = {1.f, 1.f, 1.f, 1.f}, z[4];
                if (w) ld4<E>(w + q, wo);
                ld4<float>(p, z);
                c[0] = z[0]; sn[0] = z[1]; c[1] = z[2]; sn[1] = z[3];
                ld4<float>(p + 4, z);
                c[2] = z[0]; sn[2] = z[1]; c[3] = z[2]; sn[3] = z[3];
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    o[e] = o[e] * r * wo[e];
                    if (lo) o[e] = -o[e];
                }
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int d = d0 + e;
                    if (d >= a.rot_dims) continue;
                    const bool lo = d < half;
                    const int q = k + e + (lo ? half : -half);
                    float wo = 1.0f;
                    if (w) {
                        if constexpr (sizeof(E) == 4) wo = w[q];
                        else wo = bf2f(w[q]);
                    }
                    o[e] = sp[q] * r * wo;
                    if (lo) o[e] = -o[e];
                    const float2 f = *reinterpret_cast<const float2*>(cs + 2 * (lo ? d : d - half));
                    c[e] = f.x; sn[e] = f.y;
                }
            }
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = fmaf(v[e], c[e], o[e] * sn[e]);
        }
        if (part) st4<E>(reinterpret_cast<E*>(a.kc) + (base + (size_t)hd * a.block_size) * a.dp + d0, v);
        else st4<E>(reinterpret_cast<E*>(a.q) + (size_t)t * nq + k, v);
    }
}

template <typename E, bool WIDE>
static int qkv_write_launch(const omni_qkv_write& a, size_t lds, hipStream_t st) {
    if (lds > 60 * 1024) {
        static const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(qkv_write_kernel<E, WIDE>), hipFuncAttributeMaxDynamicSharedMemorySize, 156 * 1024);
        if (e != hipSuccess) { omni_set_error("omni_qkv_write: LDS attribute: %s", hipGetErrorString(e)); return OMNI_EHIP; }
    }
    // parts in launch order: queries, (keys and values, of a layer with its own), (gate): a missing part in the middle starts and leaves
    const int parts = a.gate ? 3 : (a.kc ? 2 : 1);
    hipLaunchKernelGGL((qkv_write_kernel<E, WIDE>), dim3(a.T, parts), dim3(DR_THREADS), lds, st, a);
    OMNI_CHECK_LAUNCH("omni_qkv_write");
    return OMNI_OK;
}

extern "C" int omni_qkv_write_run(const omni_qkv_write* p, void* stream) {
    OMNI_CHECK_ARG(p && p->proj && p->q && p->row_of_tok && p->positions && (!p->kc == !p->vc), "omni_qkv_write: null pointer");
    const omni_qkv_write& a = *p;
    OMNI_CHECK_ARG(a.heads > 0 && a.kv_heads > 0 && a.heads % a.kv_heads == 0 && a.dim > 0 && a.dp >= a.dim && a.dp % 32 == 0 && a.vp > 0 && a.vp % 32 == 0,
                   "omni_qkv_write: heads %d / %d, dim %d / %d, vp %d", a.heads, a.kv_heads, a.dim, a.dp, a.vp);
    const int need = a.heads * a.dp + (a.kc ? a.kv_heads * (a.dp + a.vp) : 0) + (a.gate ? a.heads * a.vp : 0);
    OMNI_CHECK_ARG(a.ld >= need && a.ld % 4 == 0, "omni_qkv_write: ld=%d (>= %d)", a.ld, need);
    OMNI_CHECK_ARG(a.rot_dims >= 0 && a.rot_dims % 2 == 0 && a.rot_dims <= a.dim && (a.rot_dims == 0 || (a.rot && a.rot_rows > 0)), "omni_qkv_write: rot_dims=%d of %d", a.rot_dims, a.dim);
    OMNI_CHECK_ARG(!a.kc || (a.block_table && a.block_size > 0 && a.bt_stride > 0), "omni_qkv_write: block_size=%d bt_stride=%d", a.block_size, a.bt_stride);
    OMNI_CHECK_ARG(a.slabs <= OMNI_STREAM_MAX_SPLITS && (a.elem == 0 || a.elem == 1), "omni_qkv_write: slabs=%d elem=%d", a.slabs, a.elem);
    const size_t lds = (size_t)a.heads * a.dp * sizeof(float);      // (there are no more key heads than query heads)
    OMNI_CHECK_ARG(lds <= 156 * 1024, "omni_qkv_write: %d query heads of %d (a token's are staged in LDS)", a.heads, a.dp);
    if (a.T <= 0) return OMNI_OK;
    hipStream_t st = (hipStream_t)stream;
    if (a.rot_dims % 8 == 0) return a.elem ? qkv_write_launch<float, true>(a, lds, st) : qkv_write_launch<uint16_t, true>(a, lds, st);
    return a.elem ? qkv_write_launch<float, false>(a, lds, st) : qkv_write_launch<uint16_t, false>(a, lds, st);
}

// ---- a recurrence's output: norm over all heads together, times the gate.  One workgroup per token
template <typename E, int MAXC>
__global__ __launch_bounds__(DR_THREADS) void gated_norm_kernel(const omni_gated_norm a) {
    __shared__ float red[2 * DR_WAVES];
    BlockSum bsum{red, 0};
    const int t = blockIdx.x;
    float v[MAXC][4], g[MAXC][4], ss = 0.f;
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
        const int k = (c * DR_THREADS + threadIdx.x) * 4;
        v[c][0] = v[c][1] = v[c][2] = v[c][3] = 0.f;
        if (k >= a.n) continue;
        ld4<float>(a.o + (size_t)t * a.n + k, v[c]);
        if (a.slabs > 0) {
            ld4_slabs(reinterpret_cast<const float*>(a.gate) + (size_t)t * a.ld + k, a.slabs, a.slab_stride, g[c]);
#pragma unroll
            for (int e = 0; e < 4; ++e) g[c][e] = 1.0f / (1.0f + expf(-g[c][e]));
        } else {
            ld4<E>(reinterpret_cast<const E*>(a.gate) + (size_t)t * a.ld + k, g[c]);
        }
    }
#pragma unroll
    for (int c = 0; c < MAXC; ++c) ss += sq4_sum(v[c][0], v[c][1], v[c][2], v[c][3]);
    const float r = 1.0f / sqrtf(bsum(ss) / (float)a.count + a.eps);
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
        const int k = (c * DR_THREADS + threadIdx.x) * 4;
        if (k >= a.n) continue;
        float w[4];
        ld4<E>(reinterpret_cast<const E*>(a.w) + k, w);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[c][e] = v[c][e] * r * w[e] * g[c][e];
        st4<E>(reinterpret_cast<E*>(a.out) + (a.frag ? frag_off(t, k, a.n) : (size_t)t * a.n + k), v[c]);
    }
}

template <typename E>
static void gated_norm_launch(const omni_gated_norm& a, hipStream_t st) {
    const int chunks = (a.n / 4 + DR_THREADS - 1) / DR_THREADS;
    const dim3 grid(a.T), block(DR_THREADS);
    if (chunks <= 1) hipLaunchKernelGGL((gated_norm_kernel<E, 1>), grid, block, 0, st, a);
    else if (chunks <= 2) hipLaunchKernelGGL((gated_norm_kernel<E, 2>), grid, block, 0, st, a);
    else if (chunks <= 4) hipLaunchKernelGGL((gated_norm_kernel<E, 4>), grid, block, 0, st, a);
    else hipLaunchKernelGGL((gated_norm_kernel<E, 8>), grid, block, 0, st, a);
}

extern "C" int omni_gated_norm_run(const omni_gated_norm* p, void* stream) {
    OMNI_CHECK_ARG(p && p->o && p->w && p->gate && p->out, "omni_gated_norm: null pointer");
    const omni_gated_norm& a = *p;
    OMNI_CHECK_ARG(a.n > 0 && a.n % 32 == 0 && a.n <= DR_THREADS * 4 * 8 && a.count > 0 && a.count <= a.n, "omni_gated_norm: n=%d (multiple of 32, <= 8192) count=%d", a.n, a.count);
    OMNI_CHECK_ARG(a.slabs >= 0 && a.slabs <= OMNI_STREAM_MAX_SPLITS && (a.elem == 0 || (a.elem == 1 && !a.frag)), "omni_gated_norm: slabs=%d elem=%d frag=%d", a.slabs, a.elem, a.frag);
    OMNI_CHECK_ARG(a.ld >= a.n && a.ld % 4 == 0, "omni_gated_norm: ld=%d", a.ld);
    if (a.T <= 0) return OMNI_OK;
    if (a.elem) gated_norm_launch<float>(a, (hipStream_t)stream);
    else gated_norm_launch<uint16_t>(a, (hipStream_t)stream);
    OMNI_CHECK_LAUNCH("omni_gated_norm");
    return OMNI_OK;
}
