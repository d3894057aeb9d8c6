// ifa_attn_latent.hip -- latent attention: every position leaves ONE cache row [kv_rank latent c | rot_dim rotated key part] in
// 32-bit floats that all heads share; a head's unrotated key is W_uk[h] c, its value W_uv[h] c, and
//     score(i, j, h) = (q_u[i][h] . W_uk[h] c_j + q_r[i][h] . k_r[j]) * scale,   causal, ordinary softmax, optionally with a learned sink per head
// (exp(sink[h]) joins the denominator).  A layer may read the cache rows that an earlier layer has written; it then turns its queries only.
// Two forms of the same sums:
//   single tokens   the key map is absorbed into the query, qa[h] = [W_uk[h]^T q_u | q_r], which is then a query of kv_rank + rot_dim
//                   dimensions against the cache rows themselves (one shared "KV head": ifa_attention_window_f32 with the value row =
//                   the key row); the latent result goes through W_uv[h] afterwards.  The cache is read once per head, nothing is expanded.
//   prompts         keys and values of the sequence's positions are expanded by two products over the cached latents
//                   (ifa_linear_bf16w) and k_attn_latent_tile runs 128 queries of one sequence per workgroup on the fp32 matrix
//                   cores, reading the rotated key part straight from the cache rows.
// Rotation: pairs of the first rot_dims dimensions of the rotated part -- interleaved (2i, 2i + 1), or halves (i, i + rot_dims / 2) -- turn by pos * freq[i]; the angle is
// formed in double (at position 1000 one fp32 ulp of an angle is 1e-4).
#include <algorithm>
#include "ifa_host.h"
#include "ifa_f32_common.h"
#include "inferflow_amd.h"

using namespace ifa32;

namespace {

// one workgroup per row: latent normed into the cache, key part rotated into the cache, the rotated part of every query head in place
// (kv null: the queries only)
__global__ void __launch_bounds__(256) k_latent_prepare(const float *__restrict__ kv, size_t ldkv, int R, int dr, int rdims, const bf16_t *__restrict__ cw, float eps,
                                                        float *__restrict__ q, size_t ldq, int heads, int dim, const double *__restrict__ freq, float mult,
                                                        const SeqDesc *__restrict__ seqs, const int *__restrict__ row_seq, float *const *__restrict__ slot_base,
                                                        size_t cache_off, int halves)
{
    extern __shared__ float cs[];          // [rdims / 2] cos, [rdims / 2] sin
    __shared__ float red[17];
    const int t = blockIdx.x, tid = threadIdx.x, half = rdims / 2;
    const SeqDesc sd = seqs[row_seq[t]];
    const int pos = sd.pos0 + t - sd.row0;
    for (int i = tid; i < half; i += blockDim.x) {
        const double a = (double)pos * freq[i];
        cs[i] = (float)(cos(a) * (double)mult);
        cs[half + i] = (float)(sin(a) * (double)mult);
    }
    if (kv) {
        const float *kr = kv + (size_t)t * ldkv;
        float *row = slot_base[sd.slot] + cache_off + (size_t)pos * (R + dr);
        float s = 0.0f;
        for (int c = tid; c < R; c += blockDim.x) s = fmaf(kr[c], kr[c], s);
        const float rinv = 1.0f / sqrtf(block_sum(s, red) / (float)R + eps);          // (the barrier inside also publishes cs)
        for (int c = tid; c < R; c += blockDim.x) row[c] = kr[c] * rinv * bf2f(cw[c]);
        for (int i = tid; i < half; i += blockDim.x) {
            const int a = halves ? i : 2 * i, b = halves ? i + half : 2 * i + 1;
            const float u = kr[R + a], v = kr[R + b], co = cs[i], si = cs[half + i];
            row[R + a] = u * co - v * si;
            row[R + b] = v * co + u * si;
        }
        for (int c = rdims + tid; c < dr; c += blockDim.x) row[R + c] = kr[R + c];
    } else __syncthreads();
    float *qr = q + (size_t)t * ldq;
    for (int e = tid; e < heads * half; e += blockDim.x) {
        const int h = e / half, i = e % half;
        float *p = qr + (size_t)h * (dim + dr) + dim + (halves ? i : 2 * i);
        const int step = halves ? half : 1;
        const float u = p[0], v = p[step], co = cs[i], si = cs[half + i];
        p[0] = u * co - v * si;
        p[step] = v * co + u * si;
    }
}

// grid (rows, heads, chunks of 64 latent channels), four waves: qa[t][h][r] = sum_d q_u[d] W_uk[h * dim + d][r].  Lane = channel r (the
// matrix rows are read coalesced), wave w sums a quarter of the d range, the quarters meet in LDS.  Chunk 0 also copies q_r behind.
__global__ void __launch_bounds__(256) k_latent_absorb_q(const float *__restrict__ q, size_t ldq, int dim, int dr, int R, const bf16_t *__restrict__ wuk,
                                                         float *__restrict__ qa, size_t ldqa)
{
    __shared__ float part[4][64];
    const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const float *qh = q + (size_t)t * ldq + (size_t)h * (dim + dr);
    float *out = qa + (size_t)t * ldqa + (size_t)h * (R + dr);
    const int r = blockIdx.z * 64 + lane, dq = (dim + 3) / 4, d0 = wave * dq, d1 = min(dim, d0 + dq);
    const bf16_t *w = wuk + (size_t)h * dim * R + r;
    float acc = 0.0f;
    if (r < R) {
#pragma unroll 8
        for (int d = d0; d < d1; d++) acc = fmaf(qh[d], bf2f(w[(size_t)d * R]), acc);
    }
    part[wave][lane] = acc;
    __syncthreads();
    if (wave == 0 && r < R) out[r] = (part[0][lane] + part[1][lane]) + (part[2][lane] + part[3][lane]);
    if (blockIdx.z == 0) for (int e = threadIdx.x; e < dr; e += blockDim.x) out[R + e] = qh[dim + e];
}

// grid (rows, groups of four output columns), a wave per column c = h * vdim + e: out[t][c] = gate * sum_r W_uv[c][r] ol[t][h * ld_head + r];
// the gate's argument is g[t][h] (one per head) or g[t][c] (gate_cols: one per column)
__global__ void __launch_bounds__(256) k_latent_expand_out(const float *__restrict__ ol, size_t ldol, int ld_head, int heads, int vdim, int R, const bf16_t *__restrict__ wuv,
                                                           const float *__restrict__ g, size_t ldg, int gate_cols, float *__restrict__ out, size_t ldo, int vec)
{
    const int t = blockIdx.x, lane = threadIdx.x & 63, c = blockIdx.y * 4 + (threadIdx.x >> 6);
    if (c >= heads * vdim) return;
    const int h = c / vdim;
    const float *src = ol + (size_t)t * ldol + (size_t)h * ld_head;
    const bf16_t *w = wuv + (size_t)c * R;
    float acc = 0.0f;
    if (vec) {
        for (int r = lane * 8; r < R; r += 512) {
            const uint4 wv = *reinterpret_cast<const uint4 *>(w + r);
            const float4 a0 = *reinterpret_cast<const float4 *>(src + r), a1 = *reinterpret_cast<const float4 *>(src + r + 4);
            acc = fmaf(a0.x, __uint_as_float(wv.x << 16), acc); acc = fmaf(a0.y, __uint_as_float(wv.x & 0xFFFF0000u), acc);
            acc = fmaf(a0.z, __uint_as_float(wv.y << 16), acc); acc = fmaf(a0.w, __uint_as_float(wv.y & 0xFFFF0000u), acc);
            acc = fmaf(a1.x, __uint_as_float(wv.z << 16), acc); acc = fmaf(a1.y, __uint_as_float(wv.z & 0xFFFF0000u), acc);
            acc = fmaf(a1.z, __uint_as_float(wv.w << 16), acc); acc = fmaf(a1.w, __uint_as_float(wv.w & 0xFFFF0000u), acc);
        }
    } else {
        for (int r = lane; r < R; r += 64) acc = fmaf(bf2f(w[r]), src[r], acc);
    }
    acc = wave_sum(acc);
    if (lane == 0) out[(size_t)t * ldo + c] = g ? acc * sigmoid_f(g[(size_t)t * ldg + (gate_cols ? c : h)]) : acc;
}

// ---- single tokens, absorbed form: the cache rows are keys (kv_rank + rot_dim) and values (the first kv_rank) of ONE head that all
// query heads share.  grid (rows, groups of HB heads, key shares), four waves: a wave walks chunks of 16 keys, four lanes per key for the
// scores of its HB heads (the key row is read ONCE for all of them, the queries sit in LDS), one value column per lane and CPL columns per
// lane for the weighted sums, online softmax per head; the waves meet in LDS and leave {maximum, sum, weighted values} per share, which
// k_attn_latent_rows_combine merges.  Scores, weights and sums are fp32.
struct LatRowArgs {
    const float *q; size_t ldq;                 // absorbed queries [rows][heads * (R + dr)]
    int heads, R, dr;
    float scale;
    const SeqDesc *seqs; const int *row_seq; float *const *slot_base; size_t cache_off;
    float *ws; int nsplit;                      // [rows][heads][nsplit][R + 2]
    float *out; size_t ldo;                     // [rows][heads * R]
    int vec;
    const bf16_t *sink;                         // [heads] or null
};

template <int HB, int CPL>
__global__ void __launch_bounds__(256) k_attn_latent_rows(LatRowArgs P)
{
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const int D = P.R + P.dr, dv = P.R;
    float *qs = sm;                              // [HB][D]
    float *wm = qs + HB * D, *wl = wm + 4 * HB;  // [4][HB] each
    float *wacc = wl + 4 * HB;                   // [4][HB][dv]
    const int t = blockIdx.x, h0 = blockIdx.y * HB, split = blockIdx.z, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int nh = min(HB, P.heads - h0);
    const SeqDesc sd = P.seqs[P.row_seq[t]];
    const int i = sd.pos0 + t - sd.row0, nk = i + 1;
    for (int e = tid; e < HB * D; e += blockDim.x) {
        const int hh = e / D, c = e - hh * D;
        qs[e] = hh < nh ? P.q[(size_t)t * P.ldq + (size_t)(h0 + hh) * D + c] : 0.0f;
    }
    __syncthreads();
    const float *kc = P.slot_base[sd.slot] + P.cache_off;
    float m[HB], l[HB], acc[HB][CPL];
#pragma unroll
    for (int hh = 0; hh < HB; hh++) {
        m[hh] = -INFINITY; l[hh] = 0.0f;
#pragma unroll
        for (int e = 0; e < CPL; e++) acc[hh][e] = 0.0f;
    }
    const int nchunks = (nk + 15) / 16, sub = lane & 3;
    for (int ch = split * 4 + wave; ch < nchunks; ch += 4 * P.nsplit) {
        const int vi = ch * 16 + (lane >> 2);
        const bool valid = vi < nk;
        const float *kr = kc + (size_t)(valid ? vi : i) * D;
        float s[HB];
#pragma unroll
        for (int hh = 0; hh < HB; hh++) s[hh] = 0.0f;
        if (P.vec) {
            constexpr int KB = 12;          // pieces of the key row requested side by side (a chunk is bound by the latency of its requests)
            for (int c0 = 4 * sub; c0 < D; c0 += 16 * KB) {
                float4 kv[KB];
#pragma unroll
                for (int u = 0; u < KB; u++) kv[u] = *reinterpret_cast<const float4 *>(kr + min(c0 + 16 * u, D - 4));
#pragma unroll
                for (int u = 0; u < KB; u++) {
                    const int c = c0 + 16 * u;
                    if (c < D) {
#pragma unroll
                        for (int hh = 0; hh < HB; hh++) {
                            const float4 qq = *reinterpret_cast<const float4 *>(qs + hh * D + c);
                            s[hh] = fmaf(qq.x, kv[u].x, s[hh]); s[hh] = fmaf(qq.y, kv[u].y, s[hh]); s[hh] = fmaf(qq.z, kv[u].z, s[hh]); s[hh] = fmaf(qq.w, kv[u].w, s[hh]);
                        }
                    }
                }
            }
        } else {
            for (int c = sub; c < D; c += 4) {
                const float kv = kr[c];
#pragma unroll
                for (int hh = 0; hh < HB; hh++) s[hh] = fmaf(qs[hh * D + c], kv, s[hh]);
            }
        }
        float p[HB];
#pragma unroll
        for (int hh = 0; hh < HB; hh++) {
            const float sc = valid ? quad_sum(s[hh]) * P.scale : -INFINITY;
            const float m_new = fmaxf(m[hh], wave_max(sc));          // finite: the chunk holds at least one visible key
            p[hh] = valid ? expf(sc - m_new) : 0.0f;
            const float corr = m[hh] == -INFINITY ? 0.0f : expf(m[hh] - m_new);
            l[hh] = l[hh] * corr + wave_sum(sub == 0 ? p[hh] : 0.0f);
#pragma unroll
            for (int e = 0; e < CPL; e++) acc[hh][e] *= corr;
            m[hh] = m_new;
        }
        const int cnt = min(16, nk - ch * 16);
        constexpr int JB = CPL <= 8 ? 4 : 2;          // value rows requested side by side (beyond cnt: the last one again, with weight zero)
        for (int j0 = 0; j0 < cnt; j0 += JB) {
            float v[JB][CPL];
#pragma unroll
            for (int u = 0; u < JB; u++) {
                const float *vr = kc + (size_t)min(ch * 16 + j0 + u, nk - 1) * D;
#pragma unroll
                for (int e = 0; e < CPL; e++) v[u][e] = vr[min(lane + 64 * e, dv - 1)];
            }
#pragma unroll
            for (int u = 0; u < JB; u++)
#pragma unroll
                for (int hh = 0; hh < HB; hh++) {
                    const float pj = __shfl(p[hh], 4 * (j0 + u), 64);
#pragma unroll
                    for (int e = 0; e < CPL; e++) acc[hh][e] = fmaf(pj, v[u][e], acc[hh][e]);
                }
        }
    }
#pragma unroll
    for (int hh = 0; hh < HB; hh++) {
        if (lane == 0) { wm[wave * HB + hh] = m[hh]; wl[wave * HB + hh] = l[hh]; }
#pragma unroll
        for (int e = 0; e < CPL; e++) { const int d = lane + 64 * e; if (d < dv) wacc[(size_t)(wave * HB + hh) * dv + d] = acc[hh][e]; }
    }
    __syncthreads();
    for (int hh = 0; hh < nh; hh++) {
        float M = -INFINITY;
        for (int w = 0; w < 4; w++) M = fmaxf(M, wm[w * HB + hh]);
        float L = 0.0f, f[4];
        for (int w = 0; w < 4; w++) { f[w] = wm[w * HB + hh] == -INFINITY ? 0.0f : expf(wm[w * HB + hh] - M); L += wl[w * HB + hh] * f[w]; }
        float *dst = P.ws + (((size_t)t * P.heads + h0 + hh) * P.nsplit + split) * (dv + 2);
        if (tid == 0) { dst[0] = M; dst[1] = L; }
        for (int d = tid; d < dv; d += blockDim.x) {
            float o = 0.0f;
            for (int w = 0; w < 4; w++) o = fmaf(wacc[(size_t)(w * HB + hh) * dv + d], f[w], o);
            dst[2 + d] = o;
        }
    }
}

// grid (rows, heads, chunks of 64 value columns), one wave: lane sp holds share sp's maximum and sum (at most 64 shares) for the scale
// factors; then lane = column, the shares' values read four at a time (independent requests, separate sums)
__global__ void __launch_bounds__(64) k_attn_latent_rows_combine(LatRowArgs P)
{
    const int t = blockIdx.x, h = blockIdx.y, dv = P.R, nsplit = P.nsplit, lane = threadIdx.x;
    const float *src = P.ws + ((size_t)t * P.heads + h) * nsplit * (dv + 2);
    const float m_sp = lane < nsplit ? src[(size_t)lane * (dv + 2)] : -INFINITY, l_sp = lane < nsplit ? src[(size_t)lane * (dv + 2) + 1] : 0.0f;
    const float snk = P.sink ? bf2f(P.sink[h]) : -INFINITY;
    const float M = fmaxf(snk, wave_max(m_sp));
    const float f_sp = m_sp == -INFINITY ? 0.0f : expf(m_sp - M);
    const float L = wave_sum(l_sp * f_sp) + (P.sink ? expf(snk - M) : 0.0f);
    const int d = blockIdx.z * 64 + lane;
    const float *col = src + 2 + min(d, dv - 1);
    float o0 = 0.0f, o1 = 0.0f, o2 = 0.0f, o3 = 0.0f;
    int sp = 0;
    for (; sp + 4 <= nsplit; sp += 4) {
        const float v0 = col[(size_t)sp * (dv + 2)], v1 = col[(size_t)(sp + 1) * (dv + 2)], v2 = col[(size_t)(sp + 2) * (dv + 2)], v3 = col[(size_t)(sp + 3) * (dv + 2)];
        o0 = fmaf(v0, __shfl(f_sp, sp, 64), o0); o1 = fmaf(v1, __shfl(f_sp, sp + 1, 64), o1);
        o2 = fmaf(v2, __shfl(f_sp, sp + 2, 64), o2); o3 = fmaf(v3, __shfl(f_sp, sp + 3, 64), o3);
    }
    for (; sp < nsplit; sp++) o0 = fmaf(col[(size_t)sp * (dv + 2)], __shfl(f_sp, sp, 64), o0);
    if (d < dv) P.out[(size_t)t * P.ldo + (size_t)h * dv + d] = ((o0 + o1) + (o2 + o3)) / L;
}

constexpr int LR_HB = 4, LR_MAX_SPLITS = 64;

size_t latent_rows_smem(int R, int dr) { return ((size_t)LR_HB * (R + dr) + 8 * LR_HB + (size_t)4 * LR_HB * R) * 4; }

// LDS beyond 48 KB has to be granted per kernel; `reserved` remembers the largest grant of this instantiation so that a launch
// inside a captured step does not have to ask (ifa_attention_latent_rows_reserve asks ahead)
template <int CPL>
int reserve_latent_rows(size_t smem)
{
    static size_t reserved = 48 * 1024;
    if (smem <= reserved) return IFA_OK;
    IFA_REQUIRE(smem <= 160 * 1024, "ifa_attention_latent_rows_f32: %zu bytes of LDS", smem);
    IFA_HIP_CHECK(hipFuncSetAttribute((const void *)k_attn_latent_rows<LR_HB, CPL>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem));
    reserved = smem;
    return IFA_OK;
}

int reserve_latent_rows_for(int R, int dr)
{
    const int cpl = (R + 63) / 64;
    const size_t smem = latent_rows_smem(R, dr);
    if (cpl <= 1) return reserve_latent_rows<1>(smem);
    if (cpl <= 2) return reserve_latent_rows<2>(smem);
    if (cpl <= 4) return reserve_latent_rows<4>(smem);
    if (cpl <= 8) return reserve_latent_rows<8>(smem);
    return reserve_latent_rows<16>(smem);
}

template <int CPL>
void launch_latent_rows(const LatRowArgs &P, unsigned rows, hipStream_t s)
{
    hipLaunchKernelGGL((k_attn_latent_rows<LR_HB, CPL>), dim3(rows, (unsigned)((P.heads + LR_HB - 1) / LR_HB), (unsigned)P.nsplit), dim3(256), latent_rows_smem(P.R, P.dr), s, P);
}

// ---- prompts: 128 queries of one sequence per workgroup, the keys 0 .. last query walked in blocks of 32 staged once per workgroup in
// LDS; each wave owns 32 queries, one per lane of each half, held in registers as the B operand of S^T = K Q^T; O^T += V^T P^T; both on the fp32
// matrix cores (v_mfma_f32_32x32x2_f32: scores and weights stay 32-bit).  In the transposed products a lane's accumulators hold 16 keys of ITS
// query, so the online softmax is lane-local but for one exchange between the halves of the wave and the weights are the second product's B
// operand as they lie in the accumulators.  The next block's keys and values are requested before the current one is worked on.  Key columns
// beyond dim + rot_dim and value columns beyond vdim are zero padding up to 32 NTK / 32 NTV.
typedef float f32x16l __attribute__((ext_vector_type(16)));
constexpr int LT_Q = 128, LT_K = 32;

struct LatTileArgs {
    const float *q; size_t ldq;
    int heads, dim, dr, vdim, R;
    float scale;
    const float *kx; size_t ldkx;
    const float *vx; size_t ldvx;
    const int *ctx0;
    const float *g; size_t ldg; int gate_cols;
    const SeqDesc *seqs; int n_seqs;
    float *const *slot_base; size_t cache_off;
    float *out; size_t ldo;
    int vec;
    const bf16_t *sink;          // [heads] or null
    bf16_t *out16;               // the output in bfloat16 instead
};

template <int NTK, int NTV>
__global__ void __launch_bounds__(256) k_attn_latent_tile(LatTileArgs P)
{
    constexpr int DK = 32 * NTK, DKP = DK + 1, DV = 32 * NTV, DVP = DV + 1;
    extern __shared__ float sm[];
    float *Ks = sm;                          // [32][DKP]
    float *Vs = Ks + LT_K * DKP;             // [32][DVP]
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, i = lane & 31, g = lane >> 5;
    const int h = blockIdx.x, dim = P.dim, dk = P.dim + P.dr, dv = P.vdim;
    // the head is the grid's fast index, the tiles run from the last one down: the tiles with the most key blocks start first
    int tile = (int)(gridDim.y - 1 - blockIdx.y), sq = 0;
    for (; sq < P.n_seqs; sq++) {
        const int nt = (P.seqs[sq].n + LT_Q - 1) / LT_Q;
        if (tile < nt) break;
        tile -= nt;
    }
    if (sq >= P.n_seqs) return;
    const SeqDesc sd = P.seqs[sq];
    const int r0 = sd.row0 + tile * LT_Q, nq = min(LT_Q, sd.n - tile * LT_Q), p0 = sd.pos0 + tile * LT_Q;
    const float *cache = P.slot_base[sd.slot] + P.cache_off + P.R;              // rotated key part of position j: cache + j (R + dr)
    const size_t crow = (size_t)(P.R + P.dr);
    const float *kx = P.kx + (size_t)P.ctx0[sq] * P.ldkx + (size_t)h * dim, *vx = P.vx + (size_t)P.ctx0[sq] * P.ldvx + (size_t)h * dv;
    const int nq_w = min(32, max(0, nq - 32 * wave));             // queries of this wave
    const int qlo = p0 + 32 * wave, qhi = qlo + nq_w - 1;          // their positions
    const int p_last = p0 + nq - 1, nb = p_last / LT_K + 1;
    // the waves' queries in turn through the key buffer into registers: lane (i, g) takes the elements 2 s + g of query i
    float qr[16 * NTK];
#pragma unroll
    for (int w = 0; w < 4; w++) {
        for (int e = tid; e < 32 * DK; e += 256) {
            const int row = e / DK, c = e % DK;
            Ks[row * DKP + c] = 32 * w + row < nq && c < dk ? P.q[(size_t)(r0 + 32 * w + row) * P.ldq + (size_t)h * dk + c] : 0.0f;
        }
        __syncthreads();
        if (wave == w) {
#pragma unroll
            for (int s = 0; s < 16 * NTK; s++) qr[s] = Ks[i * DKP + 2 * s + g];
        }
        __syncthreads();
    }
    f32x16l o[NTV];
    float m = -INFINITY, l = 0.0f;          // of the lane's query (lane & 31)
#pragma unroll
    for (int nt = 0; nt < NTV; nt++)
#pragma unroll
        for (int r = 0; r < 16; r++) o[nt][r] = 0.0f;
    float4 kreg[NTK], vreg[NTV];
    auto fetch = [&](int b) {
        const int kb0 = b * LT_K, kc_n = min(LT_K, p_last - kb0 + 1);
#pragma unroll
        for (int u = 0; u < NTK; u++) {
            const int e = tid + 256 * u, row = e / (DK / 4), c4 = (e % (DK / 4)) * 4;
            kreg[u] = make_float4(0.f, 0.f, 0.f, 0.f);
            if (row < kc_n && c4 < dk)
                kreg[u] = *reinterpret_cast<const float4 *>(c4 < dim ? kx + (size_t)(kb0 + row) * P.ldkx + c4 : cache + (size_t)(kb0 + row) * crow + (c4 - dim));
        }
#pragma unroll
        for (int u = 0; u < NTV; u++) {
            const int e = tid + 256 * u, row = e / (DV / 4), c4 = (e % (DV / 4)) * 4;
            vreg[u] = make_float4(0.f, 0.f, 0.f, 0.f);
            if (row < kc_n && c4 < dv) vreg[u] = *reinterpret_cast<const float4 *>(vx + (size_t)(kb0 + row) * P.ldvx + c4);
        }
    };
    if (P.vec) fetch(0);
    for (int b = 0; b < nb; b++) {
        const int kb0 = b * LT_K, kc_n = min(LT_K, p_last - kb0 + 1);
        __syncthreads();                 // the previous block's K / V reads are done
        if (P.vec) {
#pragma unroll
            for (int u = 0; u < NTK; u++) {
                const int e = tid + 256 * u, row = e / (DK / 4), c4 = (e % (DK / 4)) * 4;
                float *d = Ks + row * DKP + c4;
                d[0] = kreg[u].x; d[1] = kreg[u].y; d[2] = kreg[u].z; d[3] = kreg[u].w;
            }
#pragma unroll
            for (int u = 0; u < NTV; u++) {
                const int e = tid + 256 * u, row = e / (DV / 4), c4 = (e % (DV / 4)) * 4;
                float *d = Vs + row * DVP + c4;
                d[0] = vreg[u].x; d[1] = vreg[u].y; d[2] = vreg[u].z; d[3] = vreg[u].w;
            }
            if (b + 1 < nb) fetch(b + 1);
        } else {
            for (int e = tid; e < LT_K * DK; e += 256) {
                const int row = e / DK, c = e % DK;
                Ks[row * DKP + c] = row < kc_n && c < dk ? (c < dim ? kx[(size_t)(kb0 + row) * P.ldkx + c] : cache[(size_t)(kb0 + row) * crow + (c - dim)]) : 0.0f;
            }
            for (int e = tid; e < LT_K * DV; e += 256) {
                const int row = e / DV, c = e % DV;
                Vs[row * DVP + c] = row < kc_n && c < dv ? vx[(size_t)(kb0 + row) * P.ldvx + c] : 0.0f;
            }
        }
        __syncthreads();
        if (nq_w > 0 && kb0 <= qhi) {
            f32x16l acc;
#pragma unroll
            for (int r = 0; r < 16; r++) acc[r] = 0.0f;
            const float *ka = Ks + i * DKP + g;
#pragma unroll
            for (int s = 0; s < 16 * NTK; s++) acc = __builtin_amdgcn_mfma_f32_32x32x2f32(ka[2 * s], qr[s], acc, 0, 0, 0);
            const int iq = qlo + i;
            const bool qin = i < nq_w;
            float mloc = -INFINITY;
#pragma unroll
            for (int r = 0; r < 16; r++) {
                const int kk = (r & 3) + 8 * (r >> 2) + 4 * g;
                acc[r] = qin && kk < kc_n && kb0 + kk <= iq ? acc[r] * P.scale : -INFINITY;
                mloc = fmaxf(mloc, acc[r]);
            }
            mloc = fmaxf(mloc, __shfl_xor(mloc, 32, 64));
            const float m_new = fmaxf(m, mloc);
            const float corr = m == -INFINITY ? 1.0f : expf(m - m_new);      // (m_new == -inf only while nothing was visible: sums are 0)
            float psum = 0.0f;
#pragma unroll
            for (int r = 0; r < 16; r++) { acc[r] = acc[r] == -INFINITY ? 0.0f : expf(acc[r] - m_new); psum += acc[r]; }
            l = l * corr + psum;             // (the keys of this half of the wave; the halves are added at the end)
            m = m_new;
            // step s takes keys (s & 3) + 8 (s >> 2) + 4 g
#pragma unroll
            for (int nt = 0; nt < NTV; nt++) {
#pragma unroll
                for (int r = 0; r < 16; r++) o[nt][r] *= corr;
                const float *va = Vs + 4 * g * DVP + 32 * nt + i;
#pragma unroll
                for (int s = 0; s < 16; s++)
                    o[nt] = __builtin_amdgcn_mfma_f32_32x32x2f32(va[((s & 3) + 8 * (s >> 2)) * DVP], acc[s], o[nt], 0, 0, 0);
            }
        }
    }
    // the lane holds value columns 32 nt + (r & 3) + 8 (r >> 2) + 4 g of its query
    const float ls = l + __shfl_xor(l, 32, 64);
    if (i >= nq_w) return;
    const size_t row = (size_t)(r0 + 32 * wave + i);
    const float gate = P.g && !P.gate_cols ? sigmoid_f(P.g[row * P.ldg + h]) : 1.0f;
    float sc = gate / ls;
    if (P.sink) {          // (a large sink: both sums relative to the larger of the two maxima)
        const float snk = bf2f(P.sink[h]), M = fmaxf(m, snk), f = expf(m - M);
        sc = gate * f / (ls * f + expf(snk - M));
    }
#pragma unroll
    for (int nt = 0; nt < NTV; nt++)
#pragma unroll
        for (int r = 0; r < 16; r++) {
            const int e = 32 * nt + (r & 3) + 8 * (r >> 2) + 4 * g;
            if (e < dv) {
                const size_t c = (size_t)h * dv + e;
                const float v = o[nt][r] * sc;
                const float vg = P.gate_cols ? v * sigmoid_f(P.g[row * P.ldg + c]) : v;
                if (P.out16) P.out16[row * P.ldo + c] = f2bf(vg); else P.out[row * P.ldo + c] = vg;
            }
        }
}

template <int NTK, int NTV>
int launch_latent_tile(const LatTileArgs &P, unsigned tiles, hipStream_t s)
{
    const size_t smem = (size_t)LT_K * (32 * NTK + 1 + 32 * NTV + 1) * 4;          // (at most 41 KB)
    hipLaunchKernelGGL((k_attn_latent_tile<NTK, NTV>), dim3((unsigned)P.heads, tiles), dim3(256), smem, s, P);
    IFA_LAUNCH_CHECK();
    return IFA_OK;
}

template <int NTK>
int dispatch_latent_tile_v(const LatTileArgs &P, unsigned tiles, int ntv, hipStream_t s)
{
    switch (ntv) {
    case 1: return launch_latent_tile<NTK, 1>(P, tiles, s);
    case 2: return launch_latent_tile<NTK, 2>(P, tiles, s);
    case 3: return launch_latent_tile<NTK, 3>(P, tiles, s);
    case 4: return launch_latent_tile<NTK, 4>(P, tiles, s);
    default: return ifa_fail(IFA_ERR_ARG, "ifa_attention_latent_tile_f32: value size above 128");
    }
}

} // namespace

extern "C" {

int ifa_latent_prepare_f32(const void *kv_f32, size_t ldkv, int kv_rank, int rot_dim, int rot_dims, const void *c_norm_w_bf16, float eps,
                           void *q_f32, size_t ldq, int heads, int dim, const double *freq_f64_dev, float rot_mult, const void *seqs_dev,
                           const int *row_seq_dev, size_t rows, void *const *slot_base_dev, size_t cache_off, ifa_stream stream)
{
    return ifa_latent_prepare_pairs_f32(0, kv_f32, ldkv, kv_rank, rot_dim, rot_dims, c_norm_w_bf16, eps, q_f32, ldq, heads, dim, freq_f64_dev, rot_mult, seqs_dev, row_seq_dev,
                                        rows, slot_base_dev, cache_off, stream);
}

int ifa_latent_prepare_pairs_f32(int pairing, const void *kv_f32, size_t ldkv, int kv_rank, int rot_dim, int rot_dims, const void *c_norm_w_bf16, float eps,
                                 void *q_f32, size_t ldq, int heads, int dim, const double *freq_f64_dev, float rot_mult, const void *seqs_dev,
                                 const int *row_seq_dev, size_t rows, void *const *slot_base_dev, size_t cache_off, ifa_stream stream)
{
    IFA_REQUIRE(pairing == 0 || pairing == 1, "ifa_latent_prepare_pairs_f32: pairing %d", pairing);
    IFA_REQUIRE(kv_f32 && c_norm_w_bf16 && q_f32 && freq_f64_dev && seqs_dev && row_seq_dev && slot_base_dev, "ifa_latent_prepare_f32: null pointer");
    IFA_REQUIRE(kv_rank > 0 && rot_dim >= 0 && rot_dims >= 0 && rot_dims <= rot_dim && rot_dims % 2 == 0 && heads > 0 && dim >= 0 && rows > 0
                && ldkv >= (size_t)(kv_rank + rot_dim) && ldq >= (size_t)heads * (dim + rot_dim), "ifa_latent_prepare_f32: bad shape");
    hipLaunchKernelGGL(k_latent_prepare, dim3((unsigned)rows), dim3(256), (size_t)std::max(rot_dims, 2) * 4, ifa_s(stream), (const float *)kv_f32, ldkv, kv_rank, rot_dim,
                       rot_dims, (const bf16_t *)c_norm_w_bf16, eps, (float *)q_f32, ldq, heads, dim, freq_f64_dev, rot_mult, (const SeqDesc *)seqs_dev, row_seq_dev,
                       (float *const *)slot_base_dev, cache_off, pairing);
    IFA_LAUNCH_CHECK();
    return IFA_OK;
}

int ifa_latent_rotate_q_f32(int pairing, int rot_dim, int rot_dims, void *q_f32, size_t ldq, int heads, int dim, const double *freq_f64_dev, float rot_mult,
                            const void *seqs_dev, const int *row_seq_dev, size_t rows, ifa_stream stream)
{
    IFA_REQUIRE(pairing == 0 || pairing == 1, "ifa_latent_rotate_q_f32: pairing %d", pairing);
    IFA_REQUIRE(q_f32 && freq_f64_dev && seqs_dev && row_seq_dev, "ifa_latent_rotate_q_f32: null pointer");
    IFA_REQUIRE(rot_dim >= 0 && rot_dims >= 0 && rot_dims <= rot_dim && rot_dims % 2 == 0 && heads > 0 && dim >= 0 && rows > 0 && ldq >= (size_t)heads * (dim + rot_dim),
                "ifa_latent_rotate_q_f32: bad shape");
    if (rot_dims == 0) return IFA_OK;
    hipLaunchKernelGGL(k_latent_prepare, dim3((unsigned)rows), dim3(256), (size_t)std::max(rot_dims, 2) * 4, ifa_s(stream), (const float *)nullptr, (size_t)0, 0, rot_dim,
                       rot_dims, (const bf16_t *)nullptr, 0.0f, (float *)q_f32, ldq, heads, dim, freq_f64_dev, rot_mult, (const SeqDesc *)seqs_dev, row_seq_dev,
                       (float *const *)nullptr, (size_t)0, pairing);
    IFA_LAUNCH_CHECK();
    return IFA_OK;
}

int ifa_latent_absorb_q_f32(const void *q_f32, size_t ldq, int heads, int dim, int rot_dim, int kv_rank, const void *w_uk_bf16, size_t rows,
                            void *qa_f32, size_t ldqa, ifa_stream stream)
{
    IFA_REQUIRE(q_f32 && w_uk_bf16 && qa_f32, "ifa_latent_absorb_q_f32: null pointer");
    IFA_REQUIRE(heads > 0 && heads < 65536 && dim > 0 && dim <= 8192 && rot_dim >= 0 && kv_rank > 0 && rows > 0 && ldq >= (size_t)heads * (dim + rot_dim)
                && ldqa >= (size_t)heads * (kv_rank + rot_dim), "ifa_latent_absorb_q_f32: bad shape");
    IFA_REQUIRE(kv_rank <= 64 * 65535, "ifa_latent_absorb_q_f32: latent of %d channels", kv_rank);
    hipLaunchKernelGGL(k_latent_absorb_q, dim3((unsigned)rows, (unsigned)heads, ifa_cdiv((size_t)kv_rank, 64)), dim3(256), 0, ifa_s(stream), (const float *)q_f32, ldq, dim,
                       rot_dim, kv_rank, (const bf16_t *)w_uk_bf16, (float *)qa_f32, ldqa);
    IFA_LAUNCH_CHECK();
    return IFA_OK;
}

int ifa_latent_expand_out_f32(const void *ol_f32, size_t ldol, int ld_head, int heads, int vdim, int kv_rank, const void *w_uv_bf16,
                              const void *g_f32, size_t ldg, size_t rows, void *out_f32, size_t ldo, ifa_stream stream)
{
    return ifa_latent_expand_out_gated_f32(0, ol_f32, ldol, ld_head, heads, vdim, kv_rank, w_uv_bf16, g_f32, ldg, rows, out_f32, ldo, stream);
}

int ifa_latent_expand_out_gated_f32(int gate_cols, const void *ol_f32, size_t ldol, int ld_head, int heads, int vdim, int kv_rank, const void *w_uv_bf16,
                                    const void *g_f32, size_t ldg, size_t rows, void *out_f32, size_t ldo, ifa_stream stream)
{
    IFA_REQUIRE(ol_f32 && w_uv_bf16 && out_f32, "ifa_latent_expand_out_f32: null pointer");
    IFA_REQUIRE(heads > 0 && heads < 65536 && vdim > 0 && kv_rank > 0 && kv_rank <= 8192 && ld_head >= kv_rank && rows > 0 && ldol >= (size_t)(heads - 1) * ld_head + kv_rank
                && ldo >= (size_t)heads * vdim && (!g_f32 || ldg >= (size_t)heads * (gate_cols ? vdim : 1)) && (!gate_cols || g_f32), "ifa_latent_expand_out_f32: bad shape");
    IFA_REQUIRE((size_t)heads * vdim <= 4 * 65535, "ifa_latent_expand_out_f32: %d x %d output columns", heads, vdim);
    // 16-byte requests: whole 8-element pieces in every matrix row, every head's part of a latent row on a 16-byte boundary
    const int vec = (kv_rank % 8 == 0 && ld_head % 4 == 0 && ldol % 4 == 0 && ((uintptr_t)ol_f32 & 15) == 0 && ((uintptr_t)w_uv_bf16 & 15) == 0) ? 1 : 0;
    hipLaunchKernelGGL(k_latent_expand_out, dim3((unsigned)rows, ifa_cdiv((size_t)heads * vdim, 4)), dim3(256), 0, ifa_s(stream), (const float *)ol_f32, ldol, ld_head,
                       heads, vdim, kv_rank, (const bf16_t *)w_uv_bf16, (const float *)g_f32, ldg, gate_cols ? 1 : 0, (float *)out_f32, ldo, vec);
    IFA_LAUNCH_CHECK();
    return IFA_OK;
}

int ifa_attention_latent_rows_f32(const void *qa_f32, size_t ldqa, int heads, int kv_rank, int rot_dim, float scale, const void *seqs_dev,
                                  const int *row_seq_dev, size_t rows, void *const *slot_base_dev, size_t cache_off, int max_keys, void *ws_f32,
                                  size_t ws_bytes, void *out_f32, size_t ldo, ifa_stream stream)
{
    return ifa_attention_latent_rows_sinks_f32(qa_f32, ldqa, heads, kv_rank, rot_dim, scale, nullptr, seqs_dev, row_seq_dev, rows, slot_base_dev, cache_off, max_keys, ws_f32,
                                               ws_bytes, out_f32, ldo, stream);
}

int ifa_attention_latent_rows_sinks_f32(const void *qa_f32, size_t ldqa, int heads, int kv_rank, int rot_dim, float scale, const void *sink_bf16, const void *seqs_dev,
                                        const int *row_seq_dev, size_t rows, void *const *slot_base_dev, size_t cache_off, int max_keys, void *ws_f32,
                                        size_t ws_bytes, void *out_f32, size_t ldo, ifa_stream stream)
{
    IFA_REQUIRE(qa_f32 && seqs_dev && row_seq_dev && slot_base_dev && ws_f32 && out_f32, "ifa_attention_latent_rows_f32: null pointer");
    IFA_REQUIRE(heads > 0 && heads < 65536 * LR_HB && kv_rank > 0 && kv_rank <= 1024 && rot_dim >= 0 && rows > 0 && rows < 65536 && max_keys >= 1
                && ldqa >= (size_t)heads * (kv_rank + rot_dim) && ldo >= (size_t)heads * kv_rank, "ifa_attention_latent_rows_f32: bad shape");
    LatRowArgs P;
    P.q = (const float *)qa_f32; P.ldq = ldqa; P.heads = heads; P.R = kv_rank; P.dr = rot_dim; P.scale = scale; P.seqs = (const SeqDesc *)seqs_dev;
    P.row_seq = row_seq_dev; P.slot_base = (float *const *)slot_base_dev; P.cache_off = cache_off; P.ws = (float *)ws_f32; P.out = (float *)out_f32; P.ldo = ldo;
    P.vec = ((kv_rank + rot_dim) % 4 == 0 && cache_off % 4 == 0) ? 1 : 0;
    P.sink = (const bf16_t *)sink_bf16;
    // key shares: 64 keys a share over the longest sequence the cache holds (the same for every step, so that a captured step replays),
    // fewer where many rows already fill the chip or the workspace is small
    int nsplit = std::min(LR_MAX_SPLITS, (max_keys + 63) / 64);
    const size_t groups = (size_t)(heads + LR_HB - 1) / LR_HB;
    while (nsplit > 1 && rows * groups * (size_t)nsplit > 2048) nsplit--;
    while (nsplit > 1 && rows * (size_t)heads * nsplit * ((size_t)kv_rank + 2) * 4 > ws_bytes) nsplit--;
    IFA_REQUIRE(rows * (size_t)heads * nsplit * ((size_t)kv_rank + 2) * 4 <= ws_bytes, "ifa_attention_latent_rows_f32: workspace of %zu bytes is too small", ws_bytes);
    P.nsplit = nsplit;
    hipStream_t s = ifa_s(stream);
    int rc;
    if ((rc = reserve_latent_rows_for(kv_rank, rot_dim))) return rc;
    const int cpl = (kv_rank + 63) / 64;
    if (cpl <= 1) launch_latent_rows<1>(P, (unsigned)rows, s);
    else if (cpl <= 2) launch_latent_rows<2>(P, (unsigned)rows, s);
    else if (cpl <= 4) launch_latent_rows<4>(P, (unsigned)rows, s);
    else if (cpl <= 8) launch_latent_rows<8>(P, (unsigned)rows, s);
    else launch_latent_rows<16>(P, (unsigned)rows, s);
    hipLaunchKernelGGL(k_attn_latent_rows_combine, dim3((unsigned)rows, (unsigned)heads, ifa_cdiv((size_t)kv_rank, 64)), dim3(64), 0, s, P);
    IFA_LAUNCH_CHECK();
    return IFA_OK;
}

int ifa_attention_latent_rows_reserve(int kv_rank, int rot_dim)
{
    IFA_REQUIRE(kv_rank > 0 && kv_rank <= 1024 && rot_dim >= 0, "ifa_attention_latent_rows_reserve: bad shape");
    return reserve_latent_rows_for(kv_rank, rot_dim);
}

int ifa_attention_latent_tile_f32(const void *q_f32, size_t ldq, int heads, int dim, int rot_dim, int vdim, int kv_rank, float scale,
                                  const void *kx_f32, size_t ldkx, const void *vx_f32, size_t ldvx, const int *ctx0_dev, const void *g_f32, size_t ldg,
                                  const void *seqs_dev, const void *seqs_host, int n_seqs, void *const *slot_base_dev, size_t cache_off,
                                  void *out_f32, size_t ldo, ifa_stream stream)
{
    return ifa_attention_latent_tile_gated_f32(0, q_f32, ldq, heads, dim, rot_dim, vdim, kv_rank, scale, kx_f32, ldkx, vx_f32, ldvx, ctx0_dev, g_f32, ldg, seqs_dev, seqs_host,
                                               n_seqs, slot_base_dev, cache_off, out_f32, ldo, stream);
}

int ifa_attention_latent_tile_gated_f32(int gate_cols, const void *q_f32, size_t ldq, int heads, int dim, int rot_dim, int vdim, int kv_rank, float scale,
                                        const void *kx_f32, size_t ldkx, const void *vx_f32, size_t ldvx, const int *ctx0_dev, const void *g_f32, size_t ldg,
                                        const void *seqs_dev, const void *seqs_host, int n_seqs, void *const *slot_base_dev, size_t cache_off,
                                        void *out_f32, size_t ldo, ifa_stream stream)
{
    return ifa_attention_latent_tile_sinks_f32(gate_cols, q_f32, ldq, heads, dim, rot_dim, vdim, kv_rank, scale, nullptr, kx_f32, ldkx, vx_f32, ldvx, ctx0_dev, g_f32, ldg,
                                               seqs_dev, seqs_host, n_seqs, slot_base_dev, cache_off, out_f32, nullptr, ldo, stream);
}

int ifa_attention_latent_tile_sinks_f32(int gate_cols, const void *q_f32, size_t ldq, int heads, int dim, int rot_dim, int vdim, int kv_rank, float scale,
                                        const void *sink_bf16, const void *kx_f32, size_t ldkx, const void *vx_f32, size_t ldvx, const int *ctx0_dev, const void *g_f32,
                                        size_t ldg, const void *seqs_dev, const void *seqs_host, int n_seqs, void *const *slot_base_dev, size_t cache_off, void *out_f32,
                                        void *out_bf16, size_t ldo, ifa_stream stream)
{
    IFA_REQUIRE(q_f32 && kx_f32 && vx_f32 && ctx0_dev && seqs_dev && seqs_host && slot_base_dev && (out_f32 || out_bf16), "ifa_attention_latent_tile_f32: null pointer");
    IFA_REQUIRE(heads > 0 && heads < 65536 && dim > 0 && rot_dim >= 0 && vdim > 0 && kv_rank > 0 && n_seqs > 0 && ldq >= (size_t)heads * (dim + rot_dim)
                && ldkx >= (size_t)heads * dim && ldvx >= (size_t)heads * vdim && ldo >= (size_t)heads * vdim && (!g_f32 || ldg >= (size_t)heads * (gate_cols ? vdim : 1)) && (!gate_cols || g_f32),
                "ifa_attention_latent_tile_f32: bad shape");
    const int ntk = (dim + rot_dim + 31) / 32, ntv = (vdim + 31) / 32;
    IFA_REQUIRE(ifa_attention_latent_tile_fits(dim, rot_dim, vdim), "ifa_attention_latent_tile_f32: heads of %d + %d key and %d value dimensions exceed the tile kernel", dim, rot_dim, vdim);
    LatTileArgs P;
    P.q = (const float *)q_f32; P.ldq = ldq; P.heads = heads; P.dim = dim; P.dr = rot_dim; P.vdim = vdim; P.R = kv_rank; P.scale = scale;
    P.kx = (const float *)kx_f32; P.ldkx = ldkx; P.vx = (const float *)vx_f32; P.ldvx = ldvx; P.ctx0 = ctx0_dev; P.g = (const float *)g_f32; P.ldg = ldg; P.gate_cols = gate_cols ? 1 : 0;
    P.sink = (const bf16_t *)sink_bf16; P.out16 = (bf16_t *)out_bf16;
    P.seqs = (const SeqDesc *)seqs_dev; P.n_seqs = n_seqs; P.slot_base = (float *const *)slot_base_dev; P.cache_off = cache_off; P.out = (float *)out_f32; P.ldo = ldo;
    // 16-byte requests: every source row and every part of a row starts on a 16-byte boundary
    P.vec = (dim % 4 == 0 && rot_dim % 4 == 0 && vdim % 4 == 0 && kv_rank % 4 == 0 && ldq % 4 == 0 && ldkx % 4 == 0 && ldvx % 4 == 0 && cache_off % 4 == 0
             && ((uintptr_t)q_f32 & 15) == 0 && ((uintptr_t)kx_f32 & 15) == 0 && ((uintptr_t)vx_f32 & 15) == 0) ? 1 : 0;
    const ifa_seq_desc *sh = (const ifa_seq_desc *)seqs_host;
    size_t tiles = 0;
    for (int q = 0; q < n_seqs; q++) tiles += ((size_t)sh[q].n + LT_Q - 1) / LT_Q;
    IFA_REQUIRE(tiles > 0 && tiles < 65536, "ifa_attention_latent_tile_f32: %zu query tiles", tiles);
    hipStream_t s = ifa_s(stream);
    switch (ntk) {
    case 1: return dispatch_latent_tile_v<1>(P, (unsigned)tiles, ntv, s);
    case 2: return dispatch_latent_tile_v<2>(P, (unsigned)tiles, ntv, s);
    case 3: return dispatch_latent_tile_v<3>(P, (unsigned)tiles, ntv, s);
    case 4: return dispatch_latent_tile_v<4>(P, (unsigned)tiles, ntv, s);
    case 5: return dispatch_latent_tile_v<5>(P, (unsigned)tiles, ntv, s);
    case 6: return dispatch_latent_tile_v<6>(P, (unsigned)tiles, ntv, s);
    default: return ifa_fail(IFA_ERR_ARG, "ifa_attention_latent_tile_f32: key size above 192");
    }
}

int ifa_attention_latent_tile_fits(int dim, int rot_dim, int vdim)
{
    const int ntk = (dim + rot_dim + 31) / 32, ntv = (vdim + 31) / 32;
    return ntk >= 1 && ntk <= 6 && ntv >= 1 && ntv <= 4 ? 1 : 0;
}

} // extern "C"
