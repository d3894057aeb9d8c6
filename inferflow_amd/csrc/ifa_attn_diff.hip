// ifa_attn_diff.hip -- differential attention over a per-sequence key / value cache in 32-bit floats: every head keeps TWO softmax maps over the
// same values, with queries and keys of its own for each; with a_m the output of map m,
//     o = a_1 - lambda a_2,     out = o / sqrt(mean(o^2) + eps) * out_scale * sigmoid(gate)        (mean over the head's vdim values)
// Position i sees the keys first_visible(i) .. i (ifa_f32_common.h: a sliding window and / or chunks of positions).  Grouped queries: head h reads
// key / value head h / (heads / kv_heads).  Cache rows: K [kv_heads][2 maps][dim], V [kv_heads][vdim]; queries [heads][2 maps][dim].
// Two forms of the same sums:
//   short steps   k_attn_diff_rows: a workgroup per (row, up to HB heads that share a key / value head, share of the keys); both maps' keys and the values
//                 are read once for all of them; k_attn_diff_combine merges the shares, takes the difference, norms and gates
//   prompts       k_attn_diff_tile: 64 queries of one sequence and one head per workgroup on the fp32 matrix cores (v_mfma_f32_32x32x2_f32), two waves per
//                 map: a wave owns 32 queries of ONE map, the keys of both maps and the values are staged once per workgroup, and the maps meet in LDS
//                 when all keys are done
// Scores, weights and sums are fp32.
#include <algorithm>
#include "ifa_host.h"
#include "ifa_f32_common.h"
#include "inferflow_amd.h"

using namespace ifa32;

namespace {

struct DiffArgs {
    const float *q; size_t ldq;                  // [rows][heads][2][dim]
    int heads, kv_heads, dim, vdim;
    float scale; int window, chunk;
    float lambda, out_scale, eps;
    const float *g; size_t ldg;                  // [rows][heads] or null
    const SeqDesc *seqs; const int *row_seq; float *const *slot_base; size_t k_off, v_off;
    float *out; size_t ldo;                      // [rows][heads * vdim]
    float *ws; int nsplit;                       // [rows][heads][nsplit][2 maps][vdim + 2]: maximum, sum, weighted values relative to the maximum
    bf16_t *out16;                               // tiled form: the output in bfloat16 instead
    int vec, n_seqs;
};

// grid (rows, groups of HB heads, key shares), four waves: a wave walks chunks of 16 keys, four lanes per key for the scores (each a quarter of
// the dot products in interleaved 16-byte pieces), one value column per lane and CPL columns per lane for the weighted sums, online softmax per
// head and map; the waves meet in LDS.
template <int HB, int CPL>
__global__ void __launch_bounds__(256) k_attn_diff_rows(DiffArgs P)
{
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const int d = P.dim, dv = P.vdim, D2 = 2 * d, group = P.heads / P.kv_heads, nb = (group + HB - 1) / HB;
    float *qs = sm;                                  // [HB][2][d]
    float *wm = qs + HB * D2, *wl = wm + 8 * HB;     // [4][HB][2] each
    float *wacc = wl + 8 * HB;                       // [4][HB][2][dv]
    const int t = blockIdx.x, kvh = (int)blockIdx.y / nb, hb = ((int)blockIdx.y % nb) * HB, h0 = kvh * group + hb, nh = min(HB, group - hb);
    const int split = blockIdx.z, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const SeqDesc sd = P.seqs[P.row_seq[t]];
    const int i = sd.pos0 + t - sd.row0, lo = first_visible(i, P.window, P.chunk), nk = i - lo + 1;
    if (split * 64 >= nk) {          // no keys for this share: an empty one (the combine does not read its values)
        if (tid < 2 * nh) {
            float *dst = P.ws + ((((size_t)t * P.heads + h0 + (tid >> 1)) * P.nsplit + split) * 2 + (tid & 1)) * (dv + 2);
            dst[0] = -INFINITY; dst[1] = 0.0f;
        }
        return;
    }
    for (int e = tid; e < HB * D2; e += blockDim.x) qs[e] = e < nh * D2 ? P.q[(size_t)t * P.ldq + (size_t)h0 * D2 + e] : 0.0f;
    __syncthreads();
    const size_t kvd = (size_t)P.kv_heads * D2, vvd = (size_t)P.kv_heads * dv;
    const float *kc = P.slot_base[sd.slot] + P.k_off + (size_t)lo * kvd + (size_t)kvh * D2;          // (key `vi` of the visible ones: row vi)
    const float *vc = P.slot_base[sd.slot] + P.v_off + (size_t)lo * vvd + (size_t)kvh * dv;
    float m[HB][2], l[HB][2], acc[HB][2][CPL];
#pragma unroll
    for (int hh = 0; hh < HB; hh++)
#pragma unroll
        for (int mp = 0; mp < 2; mp++) {
            m[hh][mp] = -INFINITY; l[hh][mp] = 0.0f;
#pragma unroll
            for (int e = 0; e < CPL; e++) acc[hh][mp][e] = 0.0f;
        }
    const int nchunks = (nk + 15) / 16, sub = lane & 3;
    for (int ch = split * 4 + wave; ch < nchunks; ch += 4 * P.nsplit) {
        const int vi = ch * 16 + (lane >> 2);
        const bool valid = vi < nk;
        const float *kr = kc + (size_t)(valid ? vi : nk - 1) * kvd;
        float s[HB][2];
#pragma unroll
        for (int hh = 0; hh < HB; hh++) s[hh][0] = s[hh][1] = 0.0f;
        if (P.vec) {
            constexpr int KB = 4;          // pieces of each map's key requested side by side
            for (int c0 = 4 * sub; c0 < d; c0 += 16 * KB) {
                float4 kv[2][KB];
#pragma unroll
                for (int mp = 0; mp < 2; mp++)
#pragma unroll
                    for (int u = 0; u < KB; u++) kv[mp][u] = *reinterpret_cast<const float4 *>(kr + mp * d + min(c0 + 16 * u, d - 4));
#pragma unroll
                for (int u = 0; u < KB; u++) {
                    const int c = c0 + 16 * u;
                    if (c < d) {
#pragma unroll
                        for (int mp = 0; mp < 2; mp++)
#pragma unroll
                            for (int hh = 0; hh < HB; hh++) {
                                const float4 qq = *reinterpret_cast<const float4 *>(qs + (2 * hh + mp) * d + c);
                                float a = s[hh][mp];
                                a = fmaf(qq.x, kv[mp][u].x, a); a = fmaf(qq.y, kv[mp][u].y, a); a = fmaf(qq.z, kv[mp][u].z, a); a = fmaf(qq.w, kv[mp][u].w, a);
                                s[hh][mp] = a;
                            }
                    }
                }
            }
        } else {
            for (int c = sub; c < d; c += 4)
#pragma unroll
                for (int mp = 0; mp < 2; mp++) {
                    const float kv = kr[mp * d + c];
#pragma unroll
                    for (int hh = 0; hh < HB; hh++) s[hh][mp] = fmaf(qs[(2 * hh + mp) * d + c], kv, s[hh][mp]);
                }
        }
        float p[HB][2];
#pragma unroll
        for (int hh = 0; hh < HB; hh++)
#pragma unroll
            for (int mp = 0; mp < 2; mp++) {
                const float sc = quad_sum(s[hh][mp]) * P.scale, x = valid ? sc : -INFINITY;
                const float m_new = fmaxf(m[hh][mp], quads_max(x));          // finite: the chunk holds at least one visible key
                p[hh][mp] = valid ? expf(x - m_new) : 0.0f;
                const float corr = m[hh][mp] == -INFINITY ? 0.0f : expf(m[hh][mp] - m_new);
                l[hh][mp] = l[hh][mp] * corr + quads_sum(p[hh][mp]);
#pragma unroll
                for (int e = 0; e < CPL; e++) acc[hh][mp][e] *= corr;
                m[hh][mp] = m_new;
            }
        const int cnt = min(16, nk - ch * 16);
        constexpr int JB = CPL <= 4 ? 4 : 2;          // value rows requested side by side (beyond cnt: the last one again, with weight zero)
        for (int j0 = 0; j0 < cnt; j0 += JB) {
            float v[JB][CPL];
#pragma unroll
            for (int u = 0; u < JB; u++) {
                const float *vr = vc + (size_t)min(ch * 16 + j0 + u, nk - 1) * vvd;
#pragma unroll
                for (int e = 0; e < CPL; e++) v[u][e] = vr[min(lane + 64 * e, dv - 1)];
            }
#pragma unroll
            for (int u = 0; u < JB; u++)
#pragma unroll
                for (int hh = 0; hh < HB; hh++)
#pragma unroll
                    for (int mp = 0; mp < 2; mp++) {
                        const float pj = __shfl(p[hh][mp], 4 * (j0 + u), 64);
#pragma unroll
                        for (int e = 0; e < CPL; e++) acc[hh][mp][e] = fmaf(pj, v[u][e], acc[hh][mp][e]);
                    }
        }
    }
#pragma unroll
    for (int hh = 0; hh < HB; hh++)
#pragma unroll
        for (int mp = 0; mp < 2; mp++) {
            const int w = (wave * HB + hh) * 2 + mp;
            if (lane == 0) { wm[w] = m[hh][mp]; wl[w] = l[hh][mp]; }
#pragma unroll
            for (int e = 0; e < CPL; e++) { const int c = lane + 64 * e; if (c < dv) wacc[(size_t)w * dv + c] = acc[hh][mp][e]; }
        }
    __syncthreads();
    for (int hm = wave; hm < 2 * nh; hm += 4) {          // (a wave per head and map)
        float M = -INFINITY;
#pragma unroll
        for (int w = 0; w < 4; w++) M = fmaxf(M, wm[w * 2 * HB + hm]);
        float L = 0.0f, f[4];
#pragma unroll
        for (int w = 0; w < 4; w++) { const float mw = wm[w * 2 * HB + hm]; f[w] = mw == -INFINITY ? 0.0f : expf(mw - M); L += wl[w * 2 * HB + hm] * f[w]; }
        float *dst = P.ws + ((((size_t)t * P.heads + h0 + (hm >> 1)) * P.nsplit + split) * 2 + (hm & 1)) * (dv + 2);
        if (lane == 0) { dst[0] = M; dst[1] = L; }
        for (int c = lane; c < dv; c += 64) {
            float o = 0.0f;
#pragma unroll
            for (int w = 0; w < 4; w++) o = fmaf(wacc[(size_t)(w * 2 * HB + hm) * dv + c], f[w], o);
            dst[2 + c] = o;
        }
    }
}

constexpr int DR_MAX_SPLITS = 64;

// grid (rows, heads), four waves: lane sp of every wave holds share sp's maxima and sums (at most 64 shares) for the scale factors of both maps; wave w
// adds up the shares w, w + 4, ..; the waves meet in LDS, where the difference is taken, normed over the head's columns and gated
__global__ void __launch_bounds__(256) k_attn_diff_combine(DiffArgs P)
{
    extern __shared__ float part[];          // [4][2][dv]
    __shared__ float red[17];
    const int t = blockIdx.x, h = blockIdx.y, dv = P.vdim, nsplit = P.nsplit, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const size_t st = (size_t)dv + 2;
    const float *src = P.ws + ((size_t)t * P.heads + h) * nsplit * 2 * st;
    float f[2];
#pragma unroll
    for (int mp = 0; mp < 2; mp++) {
        const float m_sp = lane < nsplit ? src[((size_t)lane * 2 + mp) * st] : -INFINITY, l_sp = lane < nsplit ? src[((size_t)lane * 2 + mp) * st + 1] : 0.0f;
        const float M = wave_max(m_sp), e = m_sp == -INFINITY ? 0.0f : expf(m_sp - M);
        f[mp] = e / wave_sum(l_sp * e);          // (the row sees at least itself: the sum is positive)
    }
    for (int c0 = 0; c0 < dv; c0 += 64) {          // (every lane walks every group of 64 columns: the factors come from other lanes)
        const int c = min(c0 + lane, dv - 1);
        float o1 = 0.0f, o2 = 0.0f;
        for (int s0 = wave; s0 < nsplit; s0 += 16) {          // four shares requested side by side (beyond the last: the last one, with weight zero)
            float v1[4], v2[4];
#pragma unroll
            for (int u = 0; u < 4; u++) { const float *r = src + (size_t)min(s0 + 4 * u, nsplit - 1) * 2 * st + 2 + c; v1[u] = r[0]; v2[u] = r[st]; }
#pragma unroll
            for (int u = 0; u < 4; u++) {
                const int sp = min(s0 + 4 * u, nsplit - 1);
                const float f1 = __shfl(f[0], sp, 64), f2 = __shfl(f[1], sp, 64);
                if (s0 + 4 * u < nsplit && f1 > 0.0f) o1 = fmaf(v1[u], f1, o1);          // (an empty share's values are not there)
                if (s0 + 4 * u < nsplit && f2 > 0.0f) o2 = fmaf(v2[u], f2, o2);
            }
        }
        if (c0 + lane < dv) { part[(size_t)(wave * 2) * dv + c] = o1; part[(size_t)(wave * 2 + 1) * dv + c] = o2; }
    }
    __syncthreads();
    float ss = 0.0f;
    for (int c = tid; c < dv; c += 256) {
        const float a1 = (part[c] + part[2 * dv + c]) + (part[4 * dv + c] + part[6 * dv + c]), a2 = (part[dv + c] + part[3 * dv + c]) + (part[5 * dv + c] + part[7 * dv + c]);
        const float o = a1 - P.lambda * a2;
        part[c] = o;          // (read again by this thread only)
        ss = fmaf(o, o, ss);
    }
    const float gate = P.g ? sigmoid_f(P.g[(size_t)t * P.ldg + h]) : 1.0f;
    const float r = P.out_scale * gate / sqrtf(block_sum(ss, red) / (float)dv + P.eps);
    for (int c = tid; c < dv; c += 256) P.out[(size_t)t * P.ldo + (size_t)h * dv + c] = part[c] * r;
}

// ---- prompts.  In the transposed products S^T = K Q^T and O^T += V^T P^T a lane's accumulators hold 16 keys of ITS query, so the online softmax is
// lane-local but for one exchange between the halves of the wave, and the weights are the second product's B operand as they lie in the
// accumulators.  The next block's keys and values are requested before the current one is worked on.  Key columns beyond dim and value columns beyond
// vdim are zero padding up to 32 NTK / 32 NTV.
typedef float f32x16d __attribute__((ext_vector_type(16)));
constexpr int DT_Q = 64, DT_K = 32;

template <int NTK, int NTV>
__global__ void __launch_bounds__(256) k_attn_diff_tile(DiffArgs P)
{
    constexpr int DK = 32 * NTK, DKP = DK + 1, DV = 32 * NTV, DVP = DV + 1;
    extern __shared__ float sm[];
    float *Ks = sm;                          // [2 maps][32][DKP]; the maps' exchange at the end: [64][33]
    float *Vs = Ks + 2 * DT_K * DKP;         // [32][DVP]
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, i = lane & 31, g = lane >> 5, mp = wave >> 1, part = wave & 1;
    const int h = blockIdx.x, kvh = h / (P.heads / P.kv_heads), dk = P.dim, dv = P.vdim;
    // the head is the grid's fast index, the tiles run from the last one down
    int tile = (int)(gridDim.y - 1 - blockIdx.y), sq = 0;
    for (; sq < P.n_seqs; sq++) {
        const int nt = (P.seqs[sq].n + DT_Q - 1) / DT_Q;
        if (tile < nt) break;
        tile -= nt;
    }
    if (sq >= P.n_seqs) return;
    const SeqDesc sd = P.seqs[sq];
    const int r0 = sd.row0 + tile * DT_Q, nq = min(DT_Q, sd.n - tile * DT_Q), p0 = sd.pos0 + tile * DT_Q;
    const size_t kvd = (size_t)P.kv_heads * 2 * dk, vvd = (size_t)P.kv_heads * dv;
    const float *kc = P.slot_base[sd.slot] + P.k_off + (size_t)kvh * 2 * dk, *vc = P.slot_base[sd.slot] + P.v_off + (size_t)kvh * dv;
    const int nq_w = min(32, max(0, nq - 32 * part));             // queries of this wave
    const int qlo = p0 + 32 * part, qhi = qlo + nq_w - 1;          // their positions
    const int lo_min = first_visible(p0, P.window, P.chunk), p_last = p0 + nq - 1, nb = (p_last - lo_min) / DT_K + 1;
    const int wave_lo = first_visible(qlo, P.window, P.chunk), lane_lo = first_visible(qlo + i, P.window, P.chunk);      // (first_visible never falls with the position)
    // the waves' queries in turn through the key buffer into registers: lane (i, g) takes the elements 2 s + g of query i
    float qr[16 * NTK];
#pragma unroll
    for (int w = 0; w < 4; w++) {
        for (int e = tid; e < 32 * DK; e += 256) {
            const int row = 32 * (w & 1) + e / DK, c = e % DK;
            Ks[(e / DK) * DKP + c] = row < nq && c < dk ? P.q[(size_t)(r0 + row) * P.ldq + (size_t)(2 * h + (w >> 1)) * dk + c] : 0.0f;
        }
        __syncthreads();
        if (wave == w) {
#pragma unroll
            for (int s = 0; s < 16 * NTK; s++) qr[s] = Ks[i * DKP + 2 * s + g];
        }
        __syncthreads();
    }
    f32x16d o[NTV];
    float m = -INFINITY, l = 0.0f;          // of the lane's query (lane & 31)
#pragma unroll
    for (int nt = 0; nt < NTV; nt++)
#pragma unroll
        for (int r = 0; r < 16; r++) o[nt][r] = 0.0f;
    float4 kreg[2 * NTK], vreg[NTV];
    auto fetch = [&](int b) {
        const int kb0 = lo_min + b * DT_K, kc_n = min(DT_K, p_last - kb0 + 1);
#pragma unroll
        for (int u = 0; u < 2 * NTK; u++) {          // (the first NTK pieces of a thread belong to map 1, the others to map 2)
            const int e = tid + 256 * (u % NTK), row = e / (DK / 4), c4 = (e % (DK / 4)) * 4;
            kreg[u] = make_float4(0.f, 0.f, 0.f, 0.f);
            if (row < kc_n && c4 < dk) kreg[u] = *reinterpret_cast<const float4 *>(kc + (size_t)(kb0 + row) * kvd + (u / NTK) * dk + c4);
        }
#pragma unroll
        for (int u = 0; u < NTV; u++) {
            const int e = tid + 256 * u, row = e / (DV / 4), c4 = (e % (DV / 4)) * 4;
            vreg[u] = make_float4(0.f, 0.f, 0.f, 0.f);
            if (row < kc_n && c4 < dv) vreg[u] = *reinterpret_cast<const float4 *>(vc + (size_t)(kb0 + row) * vvd + c4);
        }
    };
    if (P.vec) fetch(0);
    for (int b = 0; b < nb; b++) {
        const int kb0 = lo_min + b * DT_K, kc_n = min(DT_K, p_last - kb0 + 1);
        __syncthreads();                 // the previous block's K / V reads are done
        if (P.vec) {
#pragma unroll
            for (int u = 0; u < 2 * NTK; u++) {
                const int e = tid + 256 * (u % NTK), row = e / (DK / 4), c4 = (e % (DK / 4)) * 4;
                float *dst = Ks + ((u / NTK) * DT_K + row) * DKP + c4;
                dst[0] = kreg[u].x; dst[1] = kreg[u].y; dst[2] = kreg[u].z; dst[3] = kreg[u].w;
            }
#pragma unroll
            for (int u = 0; u < NTV; u++) {
                const int e = tid + 256 * u, row = e / (DV / 4), c4 = (e % (DV / 4)) * 4;
                float *dst = Vs + row * DVP + c4;
                dst[0] = vreg[u].x; dst[1] = vreg[u].y; dst[2] = vreg[u].z; dst[3] = vreg[u].w;
            }
            if (b + 1 < nb) fetch(b + 1);
        } else {
            for (int e = tid; e < 2 * DT_K * DK; e += 256) {
                const int row = (e / DK) % DT_K, mk = e / (DK * DT_K), c = e % DK;
                Ks[(mk * DT_K + row) * DKP + c] = row < kc_n && c < dk ? kc[(size_t)(kb0 + row) * kvd + mk * dk + c] : 0.0f;
            }
            for (int e = tid; e < DT_K * DV; e += 256) {
                const int row = e / DV, c = e % DV;
                Vs[row * DVP + c] = row < kc_n && c < dv ? vc[(size_t)(kb0 + row) * vvd + c] : 0.0f;
            }
        }
        __syncthreads();
        if (nq_w > 0 && kb0 <= qhi && kb0 + kc_n > wave_lo) {
            f32x16d acc;
#pragma unroll
            for (int r = 0; r < 16; r++) acc[r] = 0.0f;
            const float *ka = Ks + (mp * DT_K + i) * DKP + g;
#pragma unroll
            for (int s = 0; s < 16 * NTK; s++) acc = __builtin_amdgcn_mfma_f32_32x32x2f32(ka[2 * s], qr[s], acc, 0, 0, 0);
            const int iq = qlo + i;
            const bool qin = i < nq_w;
            float mloc = -INFINITY;
#pragma unroll
            for (int r = 0; r < 16; r++) {
                const int kk = (r & 3) + 8 * (r >> 2) + 4 * g, j = kb0 + kk;
                acc[r] = qin && kk < kc_n && j <= iq && j >= lane_lo ? acc[r] * P.scale : -INFINITY;
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
    // the lane holds value columns 32 nt + (r & 3) + 8 (r >> 2) + 4 g of its query; the waves of map 2 hand theirs over, 32 columns at a time
    const float ls = l + __shfl_xor(l, 32, 64), sc = ls > 0.0f ? 1.0f / ls : 0.0f;
    float *ex = Ks + (32 * part + i) * 33 + 4 * g;
    float ss = 0.0f;
#pragma unroll
    for (int nt = 0; nt < NTV; nt++) {
        __syncthreads();
        if (mp == 1) {
#pragma unroll
            for (int r = 0; r < 16; r++) ex[(r & 3) + 8 * (r >> 2)] = o[nt][r] * sc;
        }
        __syncthreads();
        if (mp == 0) {
#pragma unroll
            for (int r = 0; r < 16; r++) {
                o[nt][r] = o[nt][r] * sc - P.lambda * ex[(r & 3) + 8 * (r >> 2)];
                ss = fmaf(o[nt][r], o[nt][r], ss);          // (columns beyond vdim are zero in both maps)
            }
        }
    }
    if (mp != 0) return;
    ss += __shfl_xor(ss, 32, 64);
    if (i >= nq_w) return;
    const size_t row = (size_t)(r0 + 32 * part + i);
    const float gate = P.g ? sigmoid_f(P.g[row * P.ldg + h]) : 1.0f;
    const float rs = P.out_scale * gate / sqrtf(ss / (float)dv + P.eps);
    float *dst = P.out + row * P.ldo + (size_t)h * dv;
    if (P.out16) {
        bf16_t *d16 = P.out16 + row * P.ldo + (size_t)h * dv;
#pragma unroll
        for (int nt = 0; nt < NTV; nt++)
#pragma unroll
            for (int r = 0; r < 16; r++) {
                const int c = 32 * nt + (r & 3) + 8 * (r >> 2) + 4 * g;
                if (c < dv) d16[c] = f2bf(o[nt][r] * rs);
            }
        return;
    }
#pragma unroll
    for (int nt = 0; nt < NTV; nt++)
#pragma unroll
        for (int r4 = 0; r4 < 4; r4++) {
            const int c = 32 * nt + 8 * r4 + 4 * g;
            if (P.vec && c < dv) *reinterpret_cast<float4 *>(dst + c) = make_float4(o[nt][4 * r4] * rs, o[nt][4 * r4 + 1] * rs, o[nt][4 * r4 + 2] * rs, o[nt][4 * r4 + 3] * rs);
            else if (!P.vec) {
#pragma unroll
                for (int r = 0; r < 4; r++) if (c + r < dv) dst[c + r] = o[nt][4 * r4 + r] * rs;
            }
        }
}

template <int NTK, int NTV>
int launch_diff_tile(const DiffArgs &P, unsigned tiles, hipStream_t s)
{
    const size_t smem = (size_t)DT_K * (2 * (32 * NTK + 1) + 32 * NTV + 1) * 4;
    if (smem > 48 * 1024) IFA_HIP_CHECK(hipFuncSetAttribute((const void *)k_attn_diff_tile<NTK, NTV>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem));
    hipLaunchKernelGGL((k_attn_diff_tile<NTK, NTV>), dim3((unsigned)P.heads, tiles), dim3(256), smem, s, P);
    IFA_LAUNCH_CHECK();
    return IFA_OK;
}

template <int NTK>
int dispatch_diff_tile_v(const DiffArgs &P, unsigned tiles, hipStream_t s)
{
    if (P.vdim <= 32) return launch_diff_tile<NTK, 1>(P, tiles, s);
    if (P.vdim <= 64) return launch_diff_tile<NTK, 2>(P, tiles, s);
    if (P.vdim <= 96) return launch_diff_tile<NTK, 3>(P, tiles, s);
    if (P.vdim <= 128) return launch_diff_tile<NTK, 4>(P, tiles, s);
    return launch_diff_tile<NTK, 8>(P, tiles, s);
}

size_t diff_rows_smem(int hb, int dim, int vdim) { return ((size_t)hb * 2 * dim + 16 * (size_t)hb + (size_t)8 * hb * vdim) * 4; }

template <int HB, int CPL>
void launch_diff_rows(const DiffArgs &P, unsigned rows, hipStream_t s)
{
    const unsigned nb = (unsigned)((P.heads / P.kv_heads + HB - 1) / HB);
    hipLaunchKernelGGL((k_attn_diff_rows<HB, CPL>), dim3(rows, (unsigned)P.kv_heads * nb, (unsigned)P.nsplit), dim3(256), diff_rows_smem(HB, P.dim, P.vdim), s, P);
}

template <int HB>
void dispatch_diff_rows_c(const DiffArgs &P, unsigned rows, hipStream_t s)
{
    if (P.vdim <= 64) launch_diff_rows<HB, 1>(P, rows, s);
    else if (P.vdim <= 128) launch_diff_rows<HB, 2>(P, rows, s);
    else launch_diff_rows<HB, 4>(P, rows, s);
}

} // namespace

extern "C" {

int ifa_attention_diff_tile_fits(int dim, int vdim) { return dim >= 1 && dim <= 128 && vdim >= 1 && (vdim <= 128 || (vdim > 192 && vdim <= 256)) ? 1 : 0; }

int ifa_attention_diff_f32(const void *q_f32, size_t ldq, int heads, int kv_heads, int dim, int vdim, float scale, int window, int chunk, float lambda, float out_scale,
                           float eps, const void *g_f32, size_t ldg, const void *seqs_dev, const int *row_seq_dev, size_t rows, void *const *slot_base_dev, size_t k_off,
                           size_t v_off, void *out_f32, void *out_bf16, size_t ldo, const void *seqs_host, int n_seqs, int tile_min_rows, int max_keys, void *ws_f32,
                           size_t ws_bytes, ifa_stream stream)
{
    IFA_REQUIRE(q_f32 && seqs_dev && row_seq_dev && slot_base_dev && (out_f32 || out_bf16) && seqs_host, "ifa_attention_diff_f32: null pointer");
    IFA_REQUIRE(heads > 0 && heads < 65536 && kv_heads > 0 && heads % kv_heads == 0 && dim > 0 && dim <= 1024 && vdim > 0 && vdim <= 1024 && rows > 0 && window >= 0 && chunk >= 0
                && n_seqs > 0, "ifa_attention_diff_f32: bad shape (%d / %d heads of %d / %d)", heads, kv_heads, dim, vdim);
    IFA_REQUIRE(ldq >= (size_t)heads * 2 * dim && ldo >= (size_t)heads * vdim && (!g_f32 || ldg >= (size_t)heads), "ifa_attention_diff_f32: row strides too small");
    DiffArgs P;
    P.q = (const float *)q_f32; P.ldq = ldq; P.heads = heads; P.kv_heads = kv_heads; P.dim = dim; P.vdim = vdim; P.scale = scale; P.window = window; P.chunk = chunk;
    P.lambda = lambda; P.out_scale = out_scale; P.eps = eps; P.g = (const float *)g_f32; P.ldg = ldg; P.seqs = (const SeqDesc *)seqs_dev; P.row_seq = row_seq_dev;
    P.slot_base = (float *const *)slot_base_dev; P.k_off = k_off; P.v_off = v_off; P.out = (float *)out_f32; P.out16 = (bf16_t *)out_bf16; P.ldo = ldo; P.ws = (float *)ws_f32; P.nsplit = 1; P.n_seqs = n_seqs;
    const ifa_seq_desc *sh = (const ifa_seq_desc *)seqs_host;
    hipStream_t s = ifa_s(stream);
    int longest = 0;
    size_t tiles = 0;
    for (int q = 0; q < n_seqs; q++) { longest = std::max(longest, sh[q].n); tiles += ((size_t)sh[q].n + DT_Q - 1) / DT_Q; }
    // 16-byte requests: every key and value head of a cache row on a 16-byte boundary (arena bases are 256-byte aligned)
    P.vec = (dim % 4 == 0 && vdim % 4 == 0 && k_off % 4 == 0 && v_off % 4 == 0 && ldo % 4 == 0 && ((uintptr_t)out_f32 & 15) == 0) ? 1 : 0;
    if (longest >= std::max(tile_min_rows, 1) && ifa_attention_diff_tile_fits(dim, vdim)) {
        IFA_REQUIRE(tiles < 65536, "ifa_attention_diff_f32: %zu query tiles in one step", tiles);
        if (dim <= 32) return dispatch_diff_tile_v<1>(P, (unsigned)tiles, s);
        if (dim <= 64) return dispatch_diff_tile_v<2>(P, (unsigned)tiles, s);
        if (dim <= 96) return dispatch_diff_tile_v<3>(P, (unsigned)tiles, s);
        return dispatch_diff_tile_v<4>(P, (unsigned)tiles, s);
    }
    IFA_REQUIRE(!out_bf16, "ifa_attention_diff_f32: a bfloat16 output comes from the tiled form only");
    // key shares: 64 keys a share over the most keys a row can see (the same for every step, so that a captured step replays), fewer where many rows
    // already fill the chip or the workspace is small
    const int group = heads / kv_heads;
    int hb = group >= 3 ? 4 : group;
    if (vdim > 256) hb = 1;
    while (hb > 1 && diff_rows_smem(hb, dim, vdim) > 48 * 1024) hb /= 2;
    long long keys = (long long)1 << 30;
    if (max_keys > 0) keys = max_keys;
    if (window > 0) keys = std::min<long long>(keys, window);
    if (chunk > 0) keys = std::min<long long>(keys, chunk);
    int nsplit = (int)std::min<long long>(DR_MAX_SPLITS, (keys + 63) / 64);
    const size_t blocks = rows * (size_t)kv_heads * ((group + hb - 1) / hb), per_share = rows * (size_t)heads * 2 * ((size_t)vdim + 2) * 4;
    while (nsplit > 1 && blocks * (size_t)nsplit > 4096) nsplit--;
    while (nsplit > 1 && per_share * nsplit > ws_bytes) nsplit--;
    IFA_REQUIRE(ws_f32 && per_share * nsplit <= ws_bytes, "ifa_attention_diff_f32: workspace of %zu bytes is too small", ws_bytes);
    IFA_REQUIRE(blocks / rows < 65536, "ifa_attention_diff_f32: %d heads", heads);
    P.nsplit = nsplit;
    if (vdim > 256) launch_diff_rows<1, 16>(P, (unsigned)rows, s);
    else if (hb == 4) dispatch_diff_rows_c<4>(P, (unsigned)rows, s);
    else if (hb == 2) dispatch_diff_rows_c<2>(P, (unsigned)rows, s);
    else dispatch_diff_rows_c<1>(P, (unsigned)rows, s);
    hipLaunchKernelGGL(k_attn_diff_combine, dim3((unsigned)rows, (unsigned)heads), dim3(256), (size_t)8 * vdim * 4, s, P);
    IFA_LAUNCH_CHECK();
    return IFA_OK;
}

} // extern "C"
