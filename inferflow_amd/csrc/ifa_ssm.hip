// ifa_ssm.hip -- the selective state space (Mamba-2) on 32-bit activations: per head a state S [state][vdim],
//     S_t = exp(-exp(A_log) dt_t) S_(t-1) + dt_t B_t x_t^T,     y_t = S_t^T C_t + D x_t,     dt = softplus(. + dt_bias),
// with x | B | C behind a short causal convolution (+ bias) and SiLU.  Heads come in groups that share B and C.
// Three forms of the same sums:
//   single tokens   k_ssm_step: convolution, step size, state update, read-out and the carried inputs of ONE token per sequence in one launch
//   prompts         chunks of 64 tokens: k_ssd_chunk leaves every chunk's own contribution to the state (and C B^T once per group),
//                   k_ssd_pass walks the chunks element by element (each chunk's entering state), k_ssd_out adds the products inside the
//                   chunk, M X with M_ij = (C_i . B_j) exp(l_i - l_j) dt_j for j <= i (l: summed log decays), to exp(l_i) C S_in -- all
//                   products on the fp32 matrix cores (v_mfma_f32_32x32x2_f32), l summed in double
//   anything else   token by token (ifa_state_scan_ssm_f32, ifa_seqmix.hip)
// The convolution's history is a ring of `taps` rows in the slot: the input of position p lives in row p % taps.  Reading positions
// p - 1 .. p - (taps - 1) never meets the row that p writes, positions before the start read as zero whatever the slot held.
#include <algorithm>
#include "ifa_host.h"
#include "ifa_f32_common.h"
#include "inferflow_amd.h"

using namespace ifa32;

namespace {

// input of channel c at row i of the step's part of a sequence (i < 0: from the ring; before position 0: zero)
__device__ __forceinline__ float conv_in(const float *__restrict__ x, size_t ldx, const SeqDesc &sd, const float *ring, int C, int taps, int i, int c)
{
    if (i >= 0) return x[(size_t)(sd.row0 + i) * ldx + c];
    const int p = sd.pos0 + i;
    return p >= 0 ? ring[(size_t)(p % taps) * C + c] : 0.0f;
}

// grid (row tiles of RT, slices of 256 channels): a thread owns one channel and slides over RT rows with the last TAPS inputs in registers
// (TAPS 0: any number of taps, every row reads its own inputs)
constexpr int CR_RT = 16;
template <int TAPS>
__global__ void __launch_bounds__(256) k_conv_ring_silu(const float *__restrict__ x, size_t ldx, int C, int taps_, const bf16_t *__restrict__ w, const bf16_t *__restrict__ bias,
                                                        const SeqDesc *__restrict__ seqs, const int *__restrict__ row_seq, int rows, float *const *__restrict__ slot_base,
                                                        size_t state_off, float *__restrict__ y, size_t ldy)
{
    const int taps = TAPS > 0 ? TAPS : taps_;
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c >= C) return;
    const int t0 = blockIdx.x * CR_RT, t1 = min(rows, t0 + CR_RT);
    const float b = bias ? bf2f(bias[c]) : 0.0f;
    float wr[TAPS > 0 ? TAPS : 1], win[TAPS > 0 ? TAPS : 1];
    if constexpr (TAPS > 0) {
#pragma unroll
        for (int j = 0; j < TAPS; j++) wr[j] = bf2f(w[(size_t)c * TAPS + j]);
    }
    int cur = -1;
    SeqDesc sd = seqs[row_seq[t0]];
    const float *ring = nullptr;
    for (int t = t0; t < t1; t++) {
        const int q = row_seq[t];
        const bool fresh = q != cur;
        if (fresh) { cur = q; sd = seqs[q]; ring = slot_base[sd.slot] + state_off; }
        const int i = t - sd.row0;
        float acc = 0.0f;
        if constexpr (TAPS > 0) {
            if (fresh) {
#pragma unroll
                for (int j = 1; j < TAPS; j++) win[j] = conv_in(x, ldx, sd, ring, C, TAPS, i - TAPS + j, c);
            }
#pragma unroll
            for (int j = 1; j < TAPS; j++) win[j - 1] = win[j];
            win[TAPS - 1] = x[(size_t)t * ldx + c];
#pragma unroll
            for (int j = 0; j < TAPS; j++) acc = fmaf(wr[j], win[j], acc);
        } else {
            for (int j = 0; j < taps; j++) acc = fmaf(bf2f(w[(size_t)c * taps + j]), conv_in(x, ldx, sd, ring, C, taps, i - taps + 1 + j, c), acc);
        }
        y[(size_t)t * ldy + c] = silu_exact(acc + b);
    }
}

// workgroups [0, gate_blocks): dt = softplus(a + dt_bias), decay = exp(-exp(A_log) dt), a thread per (row, head); the others: the ring rows of a
// sequence's last taps - 1 inputs of this step (grid.y: sequences)
__global__ void __launch_bounds__(256) k_ssm_gates_ring(const float *__restrict__ a, size_t lda, int H, int T, const bf16_t *__restrict__ A_log, const bf16_t *__restrict__ dt_bias,
                                                        float *__restrict__ dt, float *__restrict__ g, int gate_blocks, const float *__restrict__ x, size_t ldx, int C, int taps,
                                                        const SeqDesc *__restrict__ seqs, float *const *__restrict__ slot_base, size_t state_off)
{
    if ((int)blockIdx.x < gate_blocks) {
        const int idx = (blockIdx.y * gate_blocks + blockIdx.x) * 256 + threadIdx.x;
        if (idx >= T * H) return;
        const int t = idx / H, h = idx % H;
        const float d = softplus_f(a[(size_t)t * lda + h] + bf2f(dt_bias[h]));
        dt[idx] = d;
        g[idx] = expf(-expf(bf2f(A_log[h])) * d);
        return;
    }
    const int c = ((int)blockIdx.x - gate_blocks) * 256 + threadIdx.x;
    if (c >= C) return;
    const SeqDesc sd = seqs[blockIdx.y];
    float *ring = slot_base[sd.slot] + state_off;
    for (int i = max(0, sd.n - (taps - 1)); i < sd.n; i++) ring[(size_t)((sd.pos0 + i) % taps) * C + c] = x[(size_t)(sd.row0 + i) * ldx + c];
}

// ---- single tokens.  grid (rows, heads, slices of 64 value columns), eight waves: lane = column, wave w owns state rows w, w + 8, ...  The
// state is requested first; the convolution of the slice's x channels and of the group's B and C goes through LDS.  Of the workgroups that
// share B and C the group's first head writes their ring row.
struct SsmStepArgs {
    const float *xbc; size_t ldx;
    const float *dt; size_t ldd;
    int heads, groups, N, P, taps;
    const bf16_t *w, *bias, *A_log, *dt_bias, *skip;
    const SeqDesc *seqs; const int *row_seq; float *const *slot_base; size_t conv_off, state_off;
    float *out; size_t ldo;
};

template <int NR>
__global__ void __launch_bounds__(512) k_ssm_step(SsmStepArgs A)
{
    __shared__ float xs[64], Bs[256], Cs[256], part[8][64];
    const int t = blockIdx.x, h = blockIdx.y, p0 = blockIdx.z * 64, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int N = A.N, P = A.P, pc = min(64, P - p0), hpg = A.heads / A.groups, g = h / hpg;
    const SeqDesc sd = A.seqs[A.row_seq[t]];
    float *base = A.slot_base[sd.slot];
    float *S = base + A.state_off + (size_t)h * N * P + p0 + min(lane, pc - 1);
    float sv[NR];
#pragma unroll
    for (int r = 0; r < NR; r++) { const int n = wave + 8 * r; sv[r] = sd.pos0 > 0 && n < N ? S[(size_t)n * P] : 0.0f; }
    const float d = softplus_f(A.dt[(size_t)t * A.ldd + h] + bf2f(A.dt_bias[h]));
    const float dec = expf(-expf(bf2f(A.A_log[h])) * d);
    const int inner = A.heads * P, GN = A.groups * N, C = inner + 2 * GN, taps = A.taps;
    float *ring = base + A.conv_off;
    const float *xr = A.xbc + (size_t)t * A.ldx;
    const bool shared_writer = h == g * hpg && p0 == 0;
    auto item = [&](int e, float *&dst, bool &wr) -> int {          // channel of the slice's e-th input, where it goes, whether this workgroup writes its ring row
        if (e < pc) { dst = xs + e; wr = true; return h * P + p0 + e; }
        if (e < pc + N) { dst = Bs + (e - pc); wr = shared_writer; return inner + g * N + (e - pc); }
        dst = Cs + (e - pc - N); wr = shared_writer;
        return inner + GN + g * N + (e - pc - N);
    };
    if (taps == 4) {          // the usual number of taps: every request of an input at once
        for (int e = tid; e < pc + 2 * N; e += 512) {
            float *dst; bool wr;
            const int ch = item(e, dst, wr), p = sd.pos0;
            const float cur = xr[ch], h1 = ring[(size_t)((p + 3) % 4) * C + ch], h2 = ring[(size_t)((p + 2) % 4) * C + ch], h3 = ring[(size_t)((p + 1) % 4) * C + ch];
            const bf16_t *w = A.w + (size_t)ch * 4;
            const float w0 = bf2f(w[0]), w1 = bf2f(w[1]), w2 = bf2f(w[2]), w3 = bf2f(w[3]), b = A.bias ? bf2f(A.bias[ch]) : 0.0f;
            float acc = fmaf(w0, p >= 3 ? h3 : 0.0f, 0.0f);
            acc = fmaf(w1, p >= 2 ? h2 : 0.0f, acc);
            acc = fmaf(w2, p >= 1 ? h1 : 0.0f, acc);
            acc = fmaf(w3, cur, acc);
            *dst = silu_exact(acc + b);
            if (wr) ring[(size_t)(p % 4) * C + ch] = cur;
        }
    } else
    for (int e = tid; e < pc + 2 * N; e += 512) {
        float *dst; bool wr;
        const int ch = item(e, dst, wr);
        const float cur = xr[ch];
        float acc = 0.0f;
        for (int j = 0; j < taps - 1; j++) {
            const int p = sd.pos0 - (taps - 1) + j;
            acc = fmaf(bf2f(A.w[(size_t)ch * taps + j]), p >= 0 ? ring[(size_t)(p % taps) * C + ch] : 0.0f, acc);
        }
        acc = fmaf(bf2f(A.w[(size_t)ch * taps + taps - 1]), cur, acc);
        if (A.bias) acc += bf2f(A.bias[ch]);
        *dst = silu_exact(acc);
        if (wr && taps > 1) ring[(size_t)(sd.pos0 % taps) * C + ch] = cur;
    }
    __syncthreads();
    const float xv = xs[min(lane, pc - 1)], bx = d * xv;
    float o = 0.0f;
#pragma unroll
    for (int r = 0; r < NR; r++) {
        const int n = wave + 8 * r;
        if (n < N) {
            const float s = fmaf(dec, sv[r], Bs[n] * bx);
            if (lane < pc) S[(size_t)n * P] = s;
            o = fmaf(s, Cs[n], o);
        }
    }
    part[wave][lane] = o;
    __syncthreads();
    if (wave == 0 && lane < pc) {
        float y = 0.0f;
#pragma unroll
        for (int w = 0; w < 8; w++) y += part[w][lane];
        A.out[(size_t)t * A.ldo + (size_t)h * P + p0 + lane] = fmaf(bf2f(A.skip[h]), xv, y);
    }
}

// ---- prompts in chunks of 64 tokens
typedef float f32x16s __attribute__((ext_vector_type(16)));
constexpr int SC_L = 64;

struct SsdArgs {
    const float *x, *b, *c; size_t ldx, ldb, ldc;
    int heads, groups, N, P;
    const float *dt; const bf16_t *A_log, *skip;
    const SeqDesc *seqs; int n_seqs;
    float *const *slot_base; size_t state_off;
    float *st, *G, *tot;                 // [chunks][heads][N][P], [chunks][groups][64][64], [chunks][heads]
    float *out; size_t ldo;
    int vec;
};

// chunk ci of the step: its sequence and its tokens [c0, c0 + nc) there; false: beyond the last one
__device__ __forceinline__ bool find_chunk(const SsdArgs &A, int ci, SeqDesc &sd, int &c0, int &nc)
{
    for (int q = 0; q < A.n_seqs; q++) {
        sd = A.seqs[q];
        const int k = (sd.n + SC_L - 1) / SC_L;
        if (ci < k) { c0 = ci * SC_L; nc = min(SC_L, sd.n - c0); return true; }
        ci -= k;
    }
    return false;
}

// rows [r0, r0 + nc) x columns [c0, c0 + cols) of src -> LDS rows of stride ld, zero beyond nc rows and cols columns up to pad; row j times scale[j]
__device__ __forceinline__ void stage_rows(const float *__restrict__ src, size_t lds, int nc, int cols, int pad, float *dst, int ld, const float *scale, int vec)
{
    if (vec && cols % 4 == 0) {
        const int q = pad / 4;
        for (int e = threadIdx.x; e < SC_L * q; e += blockDim.x) {
            const int j = e / q, n = (e % q) * 4;
            float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
            if (j < nc && n < cols) v = *reinterpret_cast<const float4 *>(src + (size_t)j * lds + n);
            const float f = scale ? scale[j] : 1.0f;
            float *d = dst + j * ld + n;
            d[0] = v.x * f; d[1] = v.y * f; d[2] = v.z * f; d[3] = v.w * f;
        }
    } else {
        for (int e = threadIdx.x; e < SC_L * pad; e += blockDim.x) {
            const int j = e / pad, n = e % pad;
            const float v = j < nc && n < cols ? src[(size_t)j * lds + n] : 0.0f;
            dst[j * ld + n] = scale ? v * scale[j] : v;
        }
    }
}

// the chunk's summed log decays l_j (double) and its step sizes, by the first wave; the caller synchronizes
__device__ __forceinline__ void chunk_decays(const SsdArgs &A, int h, size_t row, int nc, double *l, float *dts)
{
    if (threadIdx.x < 64) {
        const int j = threadIdx.x;
        const float d = j < nc ? A.dt[(row + j) * A.heads + h] : 0.0f;
        double s = -exp((double)bf2f(A.A_log[h])) * (double)d;
        for (int o = 1; o < 64; o <<= 1) { const double u = __shfl_up(s, o, 64); if (j >= o) s += u; }
        l[j] = s; dts[j] = d;
    }
}

// grid (chunks, heads + groups, slices of 64 value columns).  Workgroup of a head: st = sum_j exp(l_last - l_j) dt_j B_j x_j^T and tot = exp(l_last).
// Workgroup of a group: G_ij = C_i . B_j for j <= i in whole 32 x 32 tiles.
__global__ void __launch_bounds__(256) k_ssd_chunk(SsdArgs A)
{
    extern __shared__ float sm[];
    __shared__ double l[SC_L];
    __shared__ float dts[SC_L], wj[SC_L];
    const int ci = blockIdx.x, hy = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, i = lane & 31, gg = lane >> 5;
    SeqDesc sd; int c0, nc;
    if (!find_chunk(A, ci, sd, c0, nc)) return;
    const size_t row = (size_t)sd.row0 + c0;
    const int N = A.N, P = A.P;
    if (hy < A.heads) {
        const int h = hy, g = h / (A.heads / A.groups), NP = (N + 31) & ~31, p0 = blockIdx.z * 64, pc = min(64, P - p0);
        float *Bs = sm, *Xs = sm + SC_L * NP;          // [64][NP], [64][64]
        chunk_decays(A, h, row, nc, l, dts);
        __syncthreads();
        if (tid < 64) wj[tid] = expf((float)(l[nc - 1] - l[tid])) * dts[tid];          // (rows beyond nc: dts is zero and l stays at l_last)
        __syncthreads();
        stage_rows(A.b + row * A.ldb + (size_t)g * N, A.ldb, nc, N, NP, Bs, NP, wj, A.vec);
        stage_rows(A.x + row * A.ldx + (size_t)h * P + p0, A.ldx, nc, pc, 64, Xs, 64, nullptr, A.vec);
        __syncthreads();
        float *st = A.st + ((size_t)ci * A.heads + h) * N * P;
        for (int tile = wave; tile < (NP / 32) * 2; tile += 4) {
            const int m0 = (tile >> 1) * 32, n0 = (tile & 1) * 32;
            if (n0 >= pc) continue;
            f32x16s acc;
#pragma unroll
            for (int r = 0; r < 16; r++) acc[r] = 0.0f;
#pragma unroll 8
            for (int s = 0; s < SC_L / 2; s++) acc = __builtin_amdgcn_mfma_f32_32x32x2f32(Bs[(2 * s + gg) * NP + m0 + i], Xs[(2 * s + gg) * 64 + n0 + i], acc, 0, 0, 0);
#pragma unroll
            for (int r = 0; r < 16; r++) {
                const int n = m0 + (r & 3) + 8 * (r >> 2) + 4 * gg;
                if (n < N && n0 + i < pc) st[(size_t)n * P + p0 + n0 + i] = acc[r];
            }
        }
        if (tid == 0 && blockIdx.z == 0) A.tot[(size_t)ci * A.heads + h] = expf((float)l[nc - 1]);
    } else {
        if (blockIdx.z) return;
        const int g = hy - A.heads, NE = (N + 1) & ~1, ld = NE + 1;
        float *Cs = sm, *Bs = sm + SC_L * ld;          // [64][NE + 1] each
        stage_rows(A.c + row * A.ldc + (size_t)g * N, A.ldc, nc, N, NE, Cs, ld, nullptr, A.vec && NE % 4 == 0);
        stage_rows(A.b + row * A.ldb + (size_t)g * N, A.ldb, nc, N, NE, Bs, ld, nullptr, A.vec && NE % 4 == 0);
        __syncthreads();
        const int ti = wave >> 1, tj = wave & 1;
        if (tj > ti) return;
        f32x16s acc;
#pragma unroll
        for (int r = 0; r < 16; r++) acc[r] = 0.0f;
        const float *ca = Cs + (32 * ti + i) * ld + gg, *ba = Bs + (32 * tj + i) * ld + gg;
#pragma unroll 8
        for (int s = 0; s < NE / 2; s++) acc = __builtin_amdgcn_mfma_f32_32x32x2f32(ca[2 * s], ba[2 * s], acc, 0, 0, 0);
        float *G = A.G + ((size_t)ci * A.groups + g) * SC_L * SC_L;
#pragma unroll
        for (int r = 0; r < 16; r++) G[(32 * ti + (r & 3) + 8 * (r >> 2) + 4 * gg) * SC_L + 32 * tj + i] = acc[r];
    }
}

// grid (slices of 256 state elements, heads, sequences), a thread per element: the chunks in order, each one's own contribution replaced by the
// state it starts from; the state behind the last one goes to the slot
__global__ void __launch_bounds__(256) k_ssd_pass(SsdArgs A)
{
    const int e = blockIdx.x * 256 + threadIdx.x, h = blockIdx.y, q = blockIdx.z;
    const size_t NP = (size_t)A.N * A.P;
    if ((size_t)e >= NP) return;
    int first = 0;
    for (int k = 0; k < q; k++) first += (A.seqs[k].n + SC_L - 1) / SC_L;
    const SeqDesc sd = A.seqs[q];
    const int cnt = (sd.n + SC_L - 1) / SC_L;
    float *slot = A.slot_base[sd.slot] + A.state_off + (size_t)h * NP + e;
    float S = sd.pos0 > 0 ? *slot : 0.0f;
    float *st = A.st + ((size_t)first * A.heads + h) * NP + e;
    const float *tot = A.tot + (size_t)first * A.heads + h;
    const size_t step = (size_t)A.heads * NP;
    constexpr int UN = 8;
    for (int c = 0; c < cnt; c += UN) {
        float loc[UN], f[UN];
#pragma unroll
        for (int u = 0; u < UN; u++) if (c + u < cnt) { loc[u] = st[(size_t)(c + u) * step]; f[u] = tot[(size_t)(c + u) * A.heads]; }
#pragma unroll
        for (int u = 0; u < UN; u++) if (c + u < cnt) { st[(size_t)(c + u) * step] = S; S = fmaf(f[u], S, loc[u]); }
    }
    *slot = S;
}

// grid (chunks, heads, slices of 64 value columns), a wave per 32 x 32 tile of the chunk's outputs
__global__ void __launch_bounds__(256) k_ssd_out(SsdArgs A)
{
    extern __shared__ float sm[];
    __shared__ double l[SC_L];
    __shared__ float dts[SC_L], el[SC_L];
    const int ci = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, i = lane & 31, gg = lane >> 5;
    SeqDesc sd; int c0, nc;
    if (!find_chunk(A, ci, sd, c0, nc)) return;
    const size_t row = (size_t)sd.row0 + c0;
    const int N = A.N, P = A.P, g = h / (A.heads / A.groups), NE = (N + 1) & ~1, ld = NE + 1, p0 = blockIdx.z * 64, pc = min(64, P - p0);
    float *Cs = sm, *Ms = Cs + SC_L * ld, *Xs = Ms + SC_L * (SC_L + 1);          // [64][NE + 1], [64][65], [64][64]
    chunk_decays(A, h, row, nc, l, dts);
    stage_rows(A.c + row * A.ldc + (size_t)g * N, A.ldc, nc, N, NE, Cs, ld, nullptr, A.vec && NE % 4 == 0);
    stage_rows(A.x + row * A.ldx + (size_t)h * P + p0, A.ldx, nc, pc, 64, Xs, 64, nullptr, A.vec);
    __syncthreads();
    if (tid < 64) el[tid] = expf((float)l[tid]);
    const float *G = A.G + ((size_t)ci * A.groups + g) * SC_L * SC_L;
    for (int e = tid; e < SC_L * SC_L; e += 256) {
        const int r = e / SC_L, j = e % SC_L;
        Ms[r * (SC_L + 1) + j] = j <= r ? G[e] * expf((float)(l[r] - l[j])) * dts[j] : 0.0f;
    }
    __syncthreads();
    const int ti = wave >> 1, n0 = (wave & 1) * 32;
    if (n0 >= pc || 32 * ti >= nc) return;
    f32x16s acc;
#pragma unroll
    for (int r = 0; r < 16; r++) acc[r] = 0.0f;
    if (sd.pos0 > 0 || c0 > 0) {          // the state the chunk starts from (zero at the start of a sequence)
        const float *S = A.st + ((size_t)ci * A.heads + h) * N * P + p0 + min(n0 + i, pc - 1);
        const float *ca = Cs + (32 * ti + i) * ld + gg;
        constexpr int UN = 16;
        for (int s0 = 0; s0 < NE / 2; s0 += UN) {
            float sv[UN];
#pragma unroll
            for (int u = 0; u < UN; u++) { const int n = 2 * (s0 + u) + gg; sv[u] = n < N ? S[(size_t)n * P] : 0.0f; }
#pragma unroll
            for (int u = 0; u < UN; u++)
                if (s0 + u < NE / 2) acc = __builtin_amdgcn_mfma_f32_32x32x2f32(ca[2 * (s0 + u)], sv[u], acc, 0, 0, 0);
        }
#pragma unroll
        for (int r = 0; r < 16; r++) acc[r] *= el[32 * ti + (r & 3) + 8 * (r >> 2) + 4 * gg];
    }
    const float *ma = Ms + (32 * ti + i) * (SC_L + 1) + gg, *xa = Xs + gg * 64 + n0 + i;
    const int ks = 16 * (ti + 1);
#pragma unroll 8
    for (int s = 0; s < ks; s++) acc = __builtin_amdgcn_mfma_f32_32x32x2f32(ma[2 * s], xa[2 * s * 64], acc, 0, 0, 0);
    const float D = bf2f(A.skip[h]);
    if (n0 + i < pc) {
#pragma unroll
        for (int r = 0; r < 16; r++) {
            const int t = 32 * ti + (r & 3) + 8 * (r >> 2) + 4 * gg;
            if (t < nc) A.out[(row + t) * A.ldo + (size_t)h * P + p0 + n0 + i] = fmaf(D, Xs[t * 64 + n0 + i], acc[r]);
        }
    }
}

// y[t][c] = v / sqrt(mean_part(v^2) + eps) * w[c], v = o[t][c] * silu(gate[t][c]): the gate in front of the norm.  grid (rows, parts or
// groups of four parts): a workgroup or a wave per part; a thread keeps its first GN_KEEP values, more are formed again
constexpr int GN_KEEP = 8;
template <bool WHOLE>      // WHOLE: one part per workgroup; else one part per wave
__global__ void __launch_bounds__(256) k_gate_groupnorm(const float *__restrict__ o, size_t ldo, int parts, int group, const bf16_t *__restrict__ w, const float *__restrict__ gate,
                                                        size_t ldg, float eps, float *__restrict__ y, size_t ldy)
{
    __shared__ float red[17];
    const int t = blockIdx.x, part = WHOLE ? blockIdx.y : blockIdx.y * (blockDim.x >> 6) + (threadIdx.x >> 6);
    const int i0 = WHOLE ? threadIdx.x : threadIdx.x & 63, step = WHOLE ? blockDim.x : 64;
    if (!WHOLE && part >= parts) return;
    const float *orow = o + (size_t)t * ldo + (size_t)part * group, *grow = gate + (size_t)t * ldg + (size_t)part * group;
    const bf16_t *wr = w + (size_t)part * group;
    float *yrow = y + (size_t)t * ldy + (size_t)part * group;
    float v[GN_KEEP], q = 0.0f;
#pragma unroll
    for (int k = 0; k < GN_KEEP; k++) { const int c = i0 + k * step; v[k] = c < group ? orow[c] * silu_exact(grow[c]) : 0.0f; q = fmaf(v[k], v[k], q); }
    for (int c = i0 + GN_KEEP * step; c < group; c += step) { const float u = orow[c] * silu_exact(grow[c]); q = fmaf(u, u, q); }
    const float r = 1.0f / sqrtf((WHOLE ? block_sum(q, red) : wave_sum(q)) / (float)group + eps);
#pragma unroll
    for (int k = 0; k < GN_KEEP; k++) { const int c = i0 + k * step; if (c < group) yrow[c] = v[k] * r * bf2f(wr[c]); }
    for (int c = i0 + GN_KEEP * step; c < group; c += step) yrow[c] = orow[c] * silu_exact(grow[c]) * r * bf2f(wr[c]);      // (y may be o: a value is read before it is written)
}

size_t al16s(size_t v) { return (v + 15) & ~(size_t)15; }

} // namespace

extern "C" {

int ifa_conv_ring_silu_f32(const void *x_f32, size_t ldx, int channels, int taps, const void *w_bf16, const void *bias_bf16, const void *seqs_dev, const int *row_seq_dev,
                           size_t rows, void *const *slot_base_dev, size_t ring_off, void *y_f32, size_t ldy, ifa_stream stream)
{
    IFA_REQUIRE(x_f32 && w_bf16 && seqs_dev && row_seq_dev && slot_base_dev && y_f32 && x_f32 != y_f32, "ifa_conv_ring_silu_f32: null pointer or y = x");
    IFA_REQUIRE(channels > 0 && taps >= 1 && taps <= 64 && rows > 0 && rows < (1u << 31) && ldx >= (size_t)channels && ldy >= (size_t)channels && channels <= 256 * 65535,
                "ifa_conv_ring_silu_f32: bad shape");
    const dim3 grid(ifa_cdiv(rows, CR_RT), ifa_cdiv((size_t)channels, 256));
#define IFA_CR(TP) hipLaunchKernelGGL(k_conv_ring_silu<TP>, grid, dim3(256), 0, ifa_s(stream), (const float *)x_f32, ldx, channels, taps, (const bf16_t *)w_bf16, \
                                      (const bf16_t *)bias_bf16, (const SeqDesc *)seqs_dev, row_seq_dev, (int)rows, (float *const *)slot_base_dev, ring_off, (float *)y_f32, ldy)
    if (taps == 2) IFA_CR(2); else if (taps == 3) IFA_CR(3); else if (taps == 4) IFA_CR(4); else IFA_CR(0);
#undef IFA_CR
    IFA_LAUNCH_CHECK();
    return IFA_OK;
}

int ifa_ssm_gates_ring_f32(const void *a_f32, size_t lda, int heads, size_t rows, const void *a_log_bf16, const void *dt_bias_bf16, void *dt_f32, void *decay_f32,
                           const void *x_f32, size_t ldx, int channels, int taps, const void *seqs_dev, int n_seqs, void *const *slot_base_dev, size_t ring_off,
                           ifa_stream stream)
{
    IFA_REQUIRE(a_f32 && a_log_bf16 && dt_bias_bf16 && dt_f32 && decay_f32 && x_f32 && seqs_dev && slot_base_dev, "ifa_ssm_gates_ring_f32: null pointer");
    IFA_REQUIRE(heads > 0 && rows > 0 && lda >= (size_t)heads && rows * (size_t)heads < (1u << 30) && channels > 0 && ldx >= (size_t)channels && taps >= 1 && taps <= 64
                && n_seqs > 0 && n_seqs < 65536, "ifa_ssm_gates_ring_f32: bad shape");
    const unsigned gb = ifa_cdiv(ifa_cdiv(rows * heads, 256), (size_t)n_seqs);          // the gates' workgroups are shared out over the grid's rows
    hipLaunchKernelGGL(k_ssm_gates_ring, dim3(gb + (taps > 1 ? ifa_cdiv((size_t)channels, 256) : 0), (unsigned)n_seqs), dim3(256), 0, ifa_s(stream), (const float *)a_f32, lda,
                       heads, (int)rows, (const bf16_t *)a_log_bf16, (const bf16_t *)dt_bias_bf16, (float *)dt_f32, (float *)decay_f32, (int)gb, (const float *)x_f32, ldx,
                       channels, taps, (const SeqDesc *)seqs_dev, (float *const *)slot_base_dev, ring_off);
    IFA_LAUNCH_CHECK();
    return IFA_OK;
}

int ifa_ssm_step_f32(const void *xbc_f32, size_t ldx, const void *dt_f32, size_t ldd, int heads, int groups, int state, int vdim, int taps, const void *conv_w_bf16,
                     const void *conv_b_bf16, const void *a_log_bf16, const void *dt_bias_bf16, const void *skip_bf16, const void *seqs_dev, const int *row_seq_dev, size_t rows,
                     void *const *slot_base_dev, size_t ring_off, size_t state_off, void *out_f32, size_t ldo, ifa_stream stream)
{
    IFA_REQUIRE(xbc_f32 && dt_f32 && conv_w_bf16 && a_log_bf16 && dt_bias_bf16 && skip_bf16 && seqs_dev && row_seq_dev && slot_base_dev && out_f32, "ifa_ssm_step_f32: null pointer");
    IFA_REQUIRE(heads > 0 && heads < 65536 && groups > 0 && heads % groups == 0 && state > 0 && state <= 256 && vdim > 0 && vdim <= 64 * 65535 && taps >= 1 && taps <= 64
                && rows > 0 && ldx >= (size_t)heads * vdim + 2 * (size_t)groups * state && ldd >= (size_t)heads && ldo >= (size_t)heads * vdim, "ifa_ssm_step_f32: bad shape");
    SsmStepArgs A;
    A.xbc = (const float *)xbc_f32; A.ldx = ldx; A.dt = (const float *)dt_f32; A.ldd = ldd; A.heads = heads; A.groups = groups; A.N = state; A.P = vdim; A.taps = taps;
    A.w = (const bf16_t *)conv_w_bf16; A.bias = (const bf16_t *)conv_b_bf16; A.A_log = (const bf16_t *)a_log_bf16; A.dt_bias = (const bf16_t *)dt_bias_bf16;
    A.skip = (const bf16_t *)skip_bf16; A.seqs = (const SeqDesc *)seqs_dev; A.row_seq = row_seq_dev; A.slot_base = (float *const *)slot_base_dev; A.conv_off = ring_off;
    A.state_off = state_off; A.out = (float *)out_f32; A.ldo = ldo;
    const dim3 grid((unsigned)rows, (unsigned)heads, ifa_cdiv((size_t)vdim, 64));
    if (state <= 32) hipLaunchKernelGGL(k_ssm_step<4>, grid, dim3(512), 0, ifa_s(stream), A);
    else if (state <= 64) hipLaunchKernelGGL(k_ssm_step<8>, grid, dim3(512), 0, ifa_s(stream), A);
    else if (state <= 128) hipLaunchKernelGGL(k_ssm_step<16>, grid, dim3(512), 0, ifa_s(stream), A);
    else hipLaunchKernelGGL(k_ssm_step<32>, grid, dim3(512), 0, ifa_s(stream), A);
    IFA_LAUNCH_CHECK();
    return IFA_OK;
}

size_t ifa_ssm_chunked_workspace_bytes(size_t chunks, int heads, int groups, int state, int vdim)
{
    return al16s(chunks * heads * (size_t)state * vdim * 4) + al16s(chunks * groups * SC_L * SC_L * 4) + al16s(chunks * heads * 4);
}

int ifa_ssm_chunked_f32(const void *x_f32, size_t ldx, const void *b_f32, size_t ldb, const void *c_f32, size_t ldc, int heads, int groups, int state, int vdim,
                        const void *dt_f32, const void *a_log_bf16, const void *skip_bf16, const void *seqs_dev, const void *seqs_host, int n_seqs, void *const *slot_base_dev,
                        size_t state_off, void *ws, size_t ws_bytes, void *out_f32, size_t ldo, ifa_stream stream)
{
    IFA_REQUIRE(x_f32 && b_f32 && c_f32 && dt_f32 && a_log_bf16 && skip_bf16 && seqs_dev && seqs_host && slot_base_dev && ws && out_f32, "ifa_ssm_chunked_f32: null pointer");
    IFA_REQUIRE(heads > 0 && groups > 0 && heads % groups == 0 && heads + groups < 65536 && state > 0 && state <= 256 && vdim > 0 && vdim <= 64 * 65535 && n_seqs > 0 && n_seqs < 65536
                && ldx >= (size_t)heads * vdim && ldb >= (size_t)groups * state && ldc >= (size_t)groups * state && ldo >= (size_t)heads * vdim, "ifa_ssm_chunked_f32: bad shape");
    const ifa_seq_desc *sh = (const ifa_seq_desc *)seqs_host;
    size_t chunks = 0;
    for (int q = 0; q < n_seqs; q++) chunks += ((size_t)sh[q].n + SC_L - 1) / SC_L;
    IFA_REQUIRE(chunks > 0 && chunks < (1u << 30) && ws_bytes >= ifa_ssm_chunked_workspace_bytes(chunks, heads, groups, state, vdim) && ((uintptr_t)ws & 15) == 0,
                "ifa_ssm_chunked_f32: workspace of %zu bytes, %zu needed", ws_bytes, ifa_ssm_chunked_workspace_bytes(chunks, heads, groups, state, vdim));
    SsdArgs A;
    A.x = (const float *)x_f32; A.b = (const float *)b_f32; A.c = (const float *)c_f32; A.ldx = ldx; A.ldb = ldb; A.ldc = ldc; A.heads = heads; A.groups = groups; A.N = state;
    A.P = vdim; A.dt = (const float *)dt_f32; A.A_log = (const bf16_t *)a_log_bf16; A.skip = (const bf16_t *)skip_bf16; A.seqs = (const SeqDesc *)seqs_dev; A.n_seqs = n_seqs;
    A.slot_base = (float *const *)slot_base_dev; A.state_off = state_off; A.out = (float *)out_f32; A.ldo = ldo;
    A.st = (float *)ws;
    A.G = (float *)((char *)ws + al16s(chunks * heads * (size_t)state * vdim * 4));
    A.tot = (float *)((char *)A.G + al16s(chunks * groups * SC_L * SC_L * 4));
    // 16-byte requests: every row of every operand, and every head's or group's part of it, on a 16-byte boundary
    A.vec = (state % 4 == 0 && vdim % 4 == 0 && ldx % 4 == 0 && ldb % 4 == 0 && ldc % 4 == 0 && (((uintptr_t)x_f32 | (uintptr_t)b_f32 | (uintptr_t)c_f32) & 15) == 0) ? 1 : 0;
    const int NP = (state + 31) & ~31, NE = (state + 1) & ~1;
    const size_t sm1 = std::max((size_t)SC_L * (NP + 64) * 4, (size_t)2 * SC_L * (NE + 1) * 4), sm3 = ((size_t)SC_L * (NE + 1) + (size_t)SC_L * (SC_L + 1) + (size_t)SC_L * 64) * 4;
    const unsigned pz = ifa_cdiv((size_t)vdim, 64);
    hipStream_t s = ifa_s(stream);
    IFA_HIP_CHECK(hipFuncSetAttribute((const void *)k_ssd_chunk, hipFuncAttributeMaxDynamicSharedMemorySize, (int)sm1));
    IFA_HIP_CHECK(hipFuncSetAttribute((const void *)k_ssd_out, hipFuncAttributeMaxDynamicSharedMemorySize, (int)sm3));
    hipLaunchKernelGGL(k_ssd_chunk, dim3((unsigned)chunks, (unsigned)(heads + groups), pz), dim3(256), sm1, s, A);
    IFA_LAUNCH_CHECK();
    hipLaunchKernelGGL(k_ssd_pass, dim3(ifa_cdiv((size_t)state * vdim, 256), (unsigned)heads, (unsigned)n_seqs), dim3(256), 0, s, A);
    IFA_LAUNCH_CHECK();
    hipLaunchKernelGGL(k_ssd_out, dim3((unsigned)chunks, (unsigned)heads, pz), dim3(256), sm3, s, A);
    IFA_LAUNCH_CHECK();
    return IFA_OK;
}

int ifa_gate_groupnorm_f32(const void *o_f32, size_t ldo, size_t rows, int channels, int groups, const void *w_bf16, const void *gate_f32, size_t ldg, float eps,
                           void *y_f32, size_t ldy, ifa_stream stream)
{
    IFA_REQUIRE(o_f32 && w_bf16 && gate_f32 && y_f32, "ifa_gate_groupnorm_f32: null pointer");
    IFA_REQUIRE(rows > 0 && rows < (1u << 31) && channels > 0 && groups > 0 && groups < 65536 && channels % groups == 0 && ldo >= (size_t)channels && ldg >= (size_t)channels
                && ldy >= (size_t)channels, "ifa_gate_groupnorm_f32: bad arguments (%d channels in %d groups)", channels, groups);
    const int group = channels / groups;
    if (group > 256)
        hipLaunchKernelGGL(k_gate_groupnorm<true>, dim3((unsigned)rows, (unsigned)groups), dim3(group > 512 ? 256 : 128), 0, ifa_s(stream), (const float *)o_f32, ldo, groups, group,
                           (const bf16_t *)w_bf16, (const float *)gate_f32, ldg, eps, (float *)y_f32, ldy);
    else
        hipLaunchKernelGGL(k_gate_groupnorm<false>, dim3((unsigned)rows, ifa_cdiv((size_t)groups, 4)), dim3(256), 0, ifa_s(stream), (const float *)o_f32, ldo, groups, group,
                           (const bf16_t *)w_bf16, (const float *)gate_f32, ldg, eps, (float *)y_f32, ldy);
    IFA_LAUNCH_CHECK();
    return IFA_OK;
}

} // extern "C"
