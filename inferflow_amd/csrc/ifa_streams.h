// ifa_streams.h -- what lies between two sub-layers of a block with several residual streams, for one row by one workgroup.  x [rows][S][cols]:
//   0. (embed not null) X_s <- embed[token] * scale for every s          (the start of the stack)
//   1. (y not null)     X_t <- sum_s mix[s][t] X_s + mult * out[t] * y    (all new streams from the old ones; mix / out null: identity / ones)
//   2. u = sum_s in[s] X_s (in null: ones);  sum_out <- u (if asked for)
//   3. (w not null)     h = u / sqrt(mean(u^2) + eps) * w
// A thread keeps its pieces of a row (16 bytes when VEC) in registers from stage 1 to stage 3; all of a row's loads are issued before the first barrier.
#pragma once
#include "ifa_f32_common.h"

namespace ifa32 {

struct StreamArgs {
    float *x; int S, cols;
    const bf16_t *embed; const int *tokens; int vocab; float scale;
    const float *y; size_t ldy; const bf16_t *mix, *out; float mult;
    const bf16_t *in, *w; float eps;
    float *h; size_t ldh; float *sum_out; size_t ldsum;
};

template <int N> __device__ __forceinline__ void st_load(const float *p, float (&v)[N])
{
    if constexpr (N == 4) { const float4 t = *reinterpret_cast<const float4 *>(p); v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w; }
    else v[0] = p[0];
}
template <int N> __device__ __forceinline__ void st_store(float *p, const float (&v)[N])
{
    if constexpr (N == 4) *reinterpret_cast<float4 *>(p) = make_float4(v[0], v[1], v[2], v[3]);
    else p[0] = v[0];
}

// lds: SMAX * SMAX + 2 SMAX + 17 floats
template <int SMAX, bool VEC>
__device__ void streams_row(const StreamArgs &P, int row, float *lds)
{
    constexpr int N = VEC ? 4 : 1, KEEP = SMAX <= 4 ? 2 : 1;
    float *red = lds, *mx = lds + 17, *ob = mx + SMAX * SMAX, *ib = ob + SMAX;
    const int S = P.S, cols = P.cols, tid = threadIdx.x, nt = blockDim.x, pieces = cols / N;
    float *xr = P.x + (size_t)row * S * cols;
    const float *yr = P.y ? P.y + (size_t)row * P.ldy : nullptr;
    float *hr = P.h ? P.h + (size_t)row * P.ldh : nullptr, *sr = P.sum_out ? P.sum_out + (size_t)row * P.ldsum : nullptr;
    const bf16_t *er = P.embed ? P.embed + (size_t)min(max(P.tokens[row], 0), P.vocab - 1) * cols : nullptr;
    float xs[KEEP][SMAX][N], yv[KEEP][N], u[KEEP][N];
    auto fetch = [&](int c, float (&xv)[SMAX][N], float (&yy)[N]) {
        if (er) {
            float v[N];
#pragma unroll
            for (int k = 0; k < N; k++) v[k] = bf2f(er[c + k]) * P.scale;
#pragma unroll
            for (int s = 0; s < SMAX; s++)
#pragma unroll
                for (int k = 0; k < N; k++) xv[s][k] = v[k];
        } else {
#pragma unroll
            for (int s = 0; s < SMAX; s++) if (s < S) st_load<N>(xr + (size_t)s * cols + c, xv[s]);
        }
        if (yr) st_load<N>(yr + c, yy);
    };
#pragma unroll
    for (int i = 0; i < KEEP; i++) { const int p = tid + i * nt; if (p < pieces) fetch(p * N, xs[i], yv[i]); }
    for (int e = tid; e < S * S; e += nt) mx[e] = P.mix ? bf2f(P.mix[e]) : (e / S == e % S ? 1.0f : 0.0f);
    for (int e = tid; e < S; e += nt) { ob[e] = (P.out ? bf2f(P.out[e]) : 1.0f) * P.mult; ib[e] = P.in ? bf2f(P.in[e]) : 1.0f; }
    __syncthreads();
    float q = 0.0f;
    auto update = [&](int c, const float (&xv)[SMAX][N], const float (&yy)[N], float (&uu)[N]) {
#pragma unroll
        for (int k = 0; k < N; k++) uu[k] = 0.0f;
#pragma unroll
        for (int t = 0; t < SMAX; t++)
            if (t < S) {
                float n[N];
                if (yr) {
#pragma unroll
                    for (int k = 0; k < N; k++) n[k] = ob[t] * yy[k];
#pragma unroll
                    for (int s = 0; s < SMAX; s++)
                        if (s < S) {
                            const float f = mx[s * S + t];
#pragma unroll
                            for (int k = 0; k < N; k++) n[k] = fmaf(f, xv[s][k], n[k]);
                        }
                } else {
#pragma unroll
                    for (int k = 0; k < N; k++) n[k] = xv[t][k];
                }
                if (yr || er) st_store<N>(xr + (size_t)t * cols + c, n);
#pragma unroll
                for (int k = 0; k < N; k++) uu[k] = fmaf(ib[t], n[k], uu[k]);
            }
        if (sr) {
#pragma unroll
            for (int k = 0; k < N; k++) sr[c + k] = uu[k];
        }
#pragma unroll
        for (int k = 0; k < N; k++) q = fmaf(uu[k], uu[k], q);
    };
#pragma unroll
    for (int i = 0; i < KEEP; i++) { const int p = tid + i * nt; if (p < pieces) update(p * N, xs[i], yv[i], u[i]); }
    for (int p = tid + KEEP * nt; p < pieces; p += nt) {          // more columns than the workgroup keeps: read back from h below
        float xv[SMAX][N], yy[N], uu[N];
        fetch(p * N, xv, yy);
        update(p * N, xv, yy, uu);
        if (P.w) {
#pragma unroll
            for (int k = 0; k < N; k++) hr[p * N + k] = uu[k];
        }
    }
    if (!P.w) return;
    const float rinv = 1.0f / sqrtf(block_sum(q, red) / (float)cols + P.eps);
    auto finish = [&](int c, float (&uu)[N]) {
#pragma unroll
        for (int k = 0; k < N; k++) uu[k] = uu[k] * rinv * bf2f(P.w[c + k]);
        st_store<N>(hr + c, uu);
    };
#pragma unroll
    for (int i = 0; i < KEEP; i++) { const int p = tid + i * nt; if (p < pieces) finish(p * N, u[i]); }
    for (int p = tid + KEEP * nt; p < pieces; p += nt) {
        float uu[N];
        st_load<N>(hr + p * N, uu);
        finish(p * N, uu);
    }
}

} // namespace ifa32
