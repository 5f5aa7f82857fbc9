// mLSTM: a matrix memory per head with exponential gates.  With the logarithms i, f of the input and forget gate and the
// running maximum m_t = max(f_t + m_(t-1), i_t),
//     S_t = e^(f_t + m_(t-1) - m_t) S_(t-1) + e^(i_t - m_t) k_t v_t^T         n_t likewise with k_t alone
//     o_t = S_t^T q_t / (max(|n_t . q_t|, e^(-m_t)) + 1e-6)
// Everything here is fp32, the matrix instructions included.  n is carried as one more column of S (with v = 1).
//
// Prompts go in chunks of 64 tokens.  The gates are scalars that do not depend on the state, so all m_t are known ahead of
// the recurrence (k_mlstm_gates).  With F_t the sum of f from a chunk's first token to t, c the token ahead of the chunk
// and L its last one,
//     S_t = e^(F_t + m_c - m_t) S_c + sum_(j <= t) e^(F_t - F_j + i_j - m_t) k_j v_j^T
// so a chunk's outputs are two products, and S_L follows from S_c with one more.  Only that last step goes through the
// chunks in order (k_mlstm_states, which leaves the state ahead of every chunk); the pair products (k_mlstm_pairs) and the
// outputs (k_mlstm_outputs) take all chunks at once.  All factors are exponentials of what is at most 0.  The sums F_t are
// formed in double: differences of them, taken inside a chunk, decide the weights of near tokens.
#include "stack.h"
#include "rows.h"

namespace lmhip {
namespace {

#define LAUNCH(kern, grid, block, lds, ...) do { \
    hipLaunchKernelGGL(kern, grid, block, lds, stream(), __VA_ARGS__); HIP_CHECK(hipGetLastError()); } while (0)

constexpr int CT = MLSTM_CHUNK;
constexpr float NONE = -3.0e38f;
static_assert(CT == 64, "a chunk is one wave's tokens in the scan of the gates and four tiles of the matrix instruction");

__device__ __forceinline__ int up4(int n) { return (n + 3) & ~3; }

// logarithms of the input and forget gate of head h at row m
__device__ __forceinline__ float2 log_gates(const MlstmRows &a, size_t m, int h)
{
    const float *c = a.cin + m * a.ldc;
    const float i = a.cap * tanhf((c[a.o_i + h] + a.bias[a.o_i + h]) / a.cap), f = a.cap * tanhf((c[a.o_f + h] + a.bias[a.o_f + h]) / a.cap);
    return make_float2(i, fminf(f, 0.f) - log1pf(expf(-fabsf(f))));
}

// the slots of the normaliser and the running maximum ahead of position p; those behind it are slot p + 1
__device__ __forceinline__ float *n_slot(const MlstmRows &a, int p, int b, int h) { return a.n + ((size_t)((p & 1) * a.r.B + b) * a.H + h) * up4(a.dim); }
__device__ __forceinline__ float *m_slot(const MlstmRows &a, int p, int b, int h) { return a.m + (size_t)((p & 1) * a.r.B + b) * a.H + h; }

// ---------------------------------------------------------------- one token

// grid (H * nb, B): nb blocks of 256 / G * RPT columns of a head's state; G lanes share a column, four dimensions each at a
// time.  LDS: q, k [dq] (dq: dim padded to 4 G)
template <int G, int RPT>
__global__ __launch_bounds__(256) void k_mlstm_token(MlstmRows a, int nb, int dq)
{
    extern __shared__ float lds[];
    __shared__ float red[16];
    constexpr int COLS = 256 / G;
    const int tid = threadIdx.x, l = tid % G, h = blockIdx.x / nb, b = blockIdx.y, j0 = (blockIdx.x % nb) * COLS * RPT + tid / G;
    const int ds = up4(a.dim), p = a.r.pos;
    float *q = lds, *k = lds + dq;
    float *Sg = a.S + ((size_t)b * a.H + h) * a.vdim * ds;
    float4 S[RPT];
#pragma unroll
    for (int r = 0; r < RPT; r++)                         // asked for first
        S[r] = p > 0 && 4 * l < ds ? *reinterpret_cast<const float4 *>(Sg + (size_t)min(j0 + r * COLS, a.vdim - 1) * ds + 4 * l) : make_float4(0.f, 0.f, 0.f, 0.f);
    const float *c = a.cin + (size_t)b * a.ldc;
    const float2 g = log_gates(a, b, h);
    const float m = p > 0 ? *m_slot(a, p, b, h) : 0.f, mn = fmaxf(g.y + m, g.x), keep = expf(g.y + m - mn), write = expf(g.x - mn);
    const float *n0 = n_slot(a, p, b, h);
    float *n1 = n_slot(a, p + 1, b, h), nq = 0.f;
    const float scale = 1.f / sqrtf((float)a.dim);
    const bool first = blockIdx.x % nb == 0;
    for (int d = tid; d < dq; d += 256) {
        const float qv = d < a.dim ? c[a.o_q + h * a.dim + d] * scale : 0.f, kv = d < a.dim ? c[a.o_k + h * a.dim + d] : 0.f;
        q[d] = qv; k[d] = kv * write;
        if (d < ds) {
            const float n = (p > 0 ? n0[d] : 0.f) * keep + kv * write;
            nq = fmaf(n, qv, nq);
            if (first) n1[d] = n;
        }
    }
    nq = block_sum(nq, red);                              // its barriers publish q and k
    if (first && tid == 0) *m_slot(a, p + 1, b, h) = mn;
    const float den = 1.f / (fmaxf(fabsf(nq), expf(-mn)) + 1e-6f);
#pragma unroll
    for (int r = 0; r < RPT; r++) {
        const int j = j0 + r * COLS, jc = min(j, a.vdim - 1), at = h * a.vdim + jc;
        float *row = Sg + (size_t)jc * ds;
        const float v = c[a.o_v + at];
        float o = 0.f;
        for (int d = 4 * l; d < ds; d += 4 * G) {
            float4 s = S[r];
            if (d >= 4 * G) s = p > 0 ? *reinterpret_cast<const float4 *>(row + d) : make_float4(0.f, 0.f, 0.f, 0.f);
            const float4 kk = *reinterpret_cast<const float4 *>(k + d), qq = *reinterpret_cast<const float4 *>(q + d);
            s.x = fmaf(kk.x, v, s.x * keep); s.y = fmaf(kk.y, v, s.y * keep); s.z = fmaf(kk.z, v, s.z * keep); s.w = fmaf(kk.w, v, s.w * keep);
            o = fmaf(s.x, qq.x, fmaf(s.y, qq.y, fmaf(s.z, qq.z, fmaf(s.w, qq.w, o))));
            if (j < a.vdim) *reinterpret_cast<float4 *>(row + d) = s;
        }
        o = G == 64 ? wave_total(o) : group_sum<G == 64 ? 32 : G>(o);
        if (l == 0 && j < a.vdim) {
            a.o[(size_t)b * a.H * a.vdim + at] = o * den;
            if (a.gate) a.gate[(size_t)b * a.H * a.vdim + at] = sigmoid(c[a.o_g + at]);
        }
    }
}

// ---------------------------------------------------------------- many tokens

// grid (H, B), block 256: a wave takes a chunk of 64 tokens, a lane one of them.  Per token: u = F - m and w = i - F as sums
// of two floats, cf = e^(F + m_c - m), wk = e^(F_L - F + i - m_L), em = e^(-m); per chunk gk = e^(F_L + m_c - m_L).
__global__ __launch_bounds__(256) void k_mlstm_gates(MlstmRows a, int chunks)
{
    __shared__ float wa[4], wb[4];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.x, b = blockIdx.y, T = a.r.T;
    const size_t base = ((size_t)b * a.H + h) * chunks * CT;
    float carry = a.r.pos > 0 ? *m_slot(a, a.r.pos, b, h) : 0.f;
    for (int t0 = 0; t0 < T; t0 += 256) {
        const int t = t0 + tid;
        float2 g = make_float2(NONE, 0.f);                // tokens past the end change nothing
        if (t < T) g = log_gates(a, (size_t)b * T + t, h);
        double F = g.y;
        float A = g.y, M = g.x;                           // m -> max(A + m, M), composed over the tokens up to the lane's
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) {
            const double Fo = __shfl_up(F, o, 64);
            const float Ao = __shfl_up(A, o, 64), Mo = __shfl_up(M, o, 64);
            if (lane >= o) { M = fmaxf(A + Mo, M); A += Ao; F += Fo; }
        }
        if (lane == 63) { wa[wave] = A; wb[wave] = M; }
        __syncthreads();
        float mc = carry;
        for (int w = 0; w < wave; w++) mc = fmaxf(wa[w] + mc, wb[w]);
        const float m = fmaxf(A + mc, M);
        for (int w = 0; w < 4; w++) carry = fmaxf(wa[w] + carry, wb[w]);
        const double FL = __shfl(F, 63, 64);
        const float mL = __shfl(m, 63, 64);
        const int ck = t0 / CT + wave;
        if (ck < chunks) {
            const size_t i = base + t;
            const double u = F - (double)m, w = (double)g.x - F;
            const float uh = (float)u, wh = (float)w;
            a.u[i] = make_float2(uh, (float)(u - (double)uh));
            a.w[i] = make_float2(wh, t < T ? (float)(w - (double)wh) : 0.f);
            a.cf[i] = expf((float)(F + (double)mc - (double)m));
            a.wk[i] = t < T ? expf((float)(FL - F + (double)g.x - (double)mL)) : 0.f;
            a.em[i] = expf(-m);
            if (lane == 63) a.gk[((size_t)b * a.H + h) * chunks + ck] = expf((float)(FL + (double)mc - (double)mL));
        }
        __syncthreads();
    }
    if (tid == 0) *m_slot(a, a.r.pos + T, b, h) = carry;
}

// four consecutive entries from column d on of a row of n, zeros behind it; vec: the rows start on 16 bytes and n % 4 == 0
__device__ __forceinline__ float4 take4(const float *row, int d, int n, bool vec)
{
    if (vec) return d < n ? *reinterpret_cast<const float4 *>(row + d) : make_float4(0.f, 0.f, 0.f, 0.f);
    float4 v;
#pragma unroll
    for (int e = 0; e < 4; e++) (&v.x)[e] = d + e < n ? row[d + e] : 0.f;
    return v;
}

// Operands in LDS for v_mfma_f32_16x16x4_f32 (A: lane -> row lane & 15; B: lane -> column lane & 15; both: reduction index
// lane >> 4; accumulator: column lane & 15, rows 4 (lane >> 4) + 0 .. 3).  The reduction may go in any order common to both.
//   by rows [row][LDR]: four reduction steps of a lane are one 16-byte read, indices 16 kb + 4 (lane >> 4) + 0 .. 3
//   by steps [index][LDS_]: sixteen rows lie side by side
constexpr int LDR = CT + 4, LDK = CT + 16;

// grid (tiles of 64 columns, tiles of 64 dimensions, H * B), block 256: a workgroup takes one 64 x 64 tile of a head's
// state (columns 0 .. vdim - 1, column vdim the normaliser) through the chunks in order, a wave a quarter of it.
__global__ __launch_bounds__(256) void k_mlstm_states(MlstmRows a, int chunks)
{
    __shared__ float Ks[CT * LDK], Vs[CT * LDK];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, r4 = lane >> 4;
    const int h = blockIdx.z % a.H, b = blockIdx.z / a.H, T = a.r.T, ds = up4(a.dim), V1 = a.vdim + 1;
    const int v0 = blockIdx.x * 64, d0 = blockIdx.y * 64, wv = v0 + (wave & 1) * 32, wd = d0 + (wave >> 1) * 32;
    const bool kvec = a.dim % 4 == 0, vvec = a.vdim % 4 == 0;
    float4v S[2][2];
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int j = 0; j < 2; j++)
#pragma unroll
            for (int x = 0; x < 4; x++) {
                const int v = wv + 16 * i + 4 * r4 + x, d = wd + 16 * j + c;
                float s = 0.f;
                if (a.r.pos > 0 && d < ds && v <= a.vdim)
                    s = v < a.vdim ? a.S[(((size_t)b * a.H + h) * a.vdim + v) * ds + d] : n_slot(a, a.r.pos, b, h)[d];
                S[i][j][x] = s;
            }
    float4 kr[4], vr[4];
    const int tok = tid >> 4, at = (tid & 15) * 4;        // four tokens of a thread, sixteen apart
    auto fetch = [&](int ck) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int t = ck * CT + tok + 16 * i;
            const float *row = a.cin + ((size_t)b * T + min(t, T - 1)) * a.ldc;
            kr[i] = take4(row + a.o_k + h * a.dim, d0 + at, a.dim, kvec);
            vr[i] = take4(row + a.o_v + h * a.vdim, v0 + at, a.vdim, vvec);
#pragma unroll
            for (int e = 0; e < 4; e++) if (v0 + at + e == a.vdim) (&vr[i].x)[e] = 1.f;
            const float w = a.wk[(((size_t)b * a.H + h) * chunks + ck) * CT + tok + 16 * i];      // 0 past the end
            kr[i].x *= w; kr[i].y *= w; kr[i].z *= w; kr[i].w *= w;
        }
    };
    fetch(0);
    for (int ck = 0; ck < chunks; ck++) {
        __syncthreads();
#pragma unroll
        for (int i = 0; i < 4; i++) {
            *reinterpret_cast<float4 *>(&Ks[(tok + 16 * i) * LDK + at]) = kr[i];
            *reinterpret_cast<float4 *>(&Vs[(tok + 16 * i) * LDK + at]) = vr[i];
        }
        __syncthreads();
        if (ck + 1 < chunks) fetch(ck + 1);
        const float g = a.gk[((size_t)b * a.H + h) * chunks + ck];
        float *out = a.Sc + (((size_t)b * chunks + ck) * a.H + h) * V1 * ds;
#pragma unroll
        for (int i = 0; i < 2; i++)
#pragma unroll
            for (int j = 0; j < 2; j++)
#pragma unroll
                for (int x = 0; x < 4; x++) {             // the state ahead of the chunk
                    const int v = wv + 16 * i + 4 * r4 + x, d = wd + 16 * j + c;
                    if (v < V1 && d < ds) out[(size_t)v * ds + d] = S[i][j][x];
                    S[i][j][x] *= g;
                }
        const float *kp = Ks + r4 * LDK + (wave >> 1) * 32 + c, *vp = Vs + r4 * LDK + (wave & 1) * 32 + c;
#pragma unroll 4
        for (int s = 0; s < CT / 4; s++) {
            float av[2], bv[2];
#pragma unroll
            for (int i = 0; i < 2; i++) { av[i] = vp[4 * s * LDK + 16 * i]; bv[i] = kp[4 * s * LDK + 16 * i]; }
#pragma unroll
            for (int i = 0; i < 2; i++)
#pragma unroll
                for (int j = 0; j < 2; j++) S[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(av[i], bv[j], S[i][j], 0, 0, 0);
        }
    }
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int j = 0; j < 2; j++)
#pragma unroll
            for (int x = 0; x < 4; x++) {
                const int v = wv + 16 * i + 4 * r4 + x, d = wd + 16 * j + c;
                if (d >= ds || v > a.vdim) continue;
                if (v < a.vdim) a.S[(((size_t)b * a.H + h) * a.vdim + v) * ds + d] = S[i][j][x];
                else n_slot(a, a.r.pos + T, b, h)[d] = S[i][j][x];
            }
}

// acc[2][2] += rows A[32 of them] x rows B[32 of them] of two LDS tiles held by rows, over 16 `blocks` of reduction indices
template <int BLOCKS>
__device__ __forceinline__ void tile_product(const float *A, const float *B, int c, int r4, float4v (&acc)[2][2])
{
#pragma unroll
    for (int kb = 0; kb < BLOCKS; kb++) {
        float4v av[2], bv[2];
#pragma unroll
        for (int i = 0; i < 2; i++) {
            av[i] = *reinterpret_cast<const float4v *>(A + (16 * i + c) * LDR + 16 * kb + 4 * r4);
            bv[i] = *reinterpret_cast<const float4v *>(B + (16 * i + c) * LDR + 16 * kb + 4 * r4);
        }
#pragma unroll
        for (int x = 0; x < 4; x++)
#pragma unroll
            for (int i = 0; i < 2; i++)
#pragma unroll
                for (int j = 0; j < 2; j++) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(av[i][x], bv[j][x], acc[i][j], 0, 0, 0);
    }
}

// grid (chunks, H, B), block 256: weights of the chunk's pairs over their denominators, P [token][token], and qf, the factor
// of the state's part of a token's output
__global__ __launch_bounds__(256) void k_mlstm_pairs(MlstmRows a, int chunks)
{
    __shared__ float Qs[CT * LDR], Ks[CT * LDR], ns[CT], sums[2][CT], qn[CT], rd[CT];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, r4 = lane >> 4;
    const int ck = blockIdx.x, h = blockIdx.y, b = blockIdx.z, T = a.r.T, ds = up4(a.dim), nt = min(CT, T - ck * CT);
    const size_t g0 = (((size_t)b * a.H + h) * chunks + ck) * CT;
    const float *nc = a.Sc + ((((size_t)b * chunks + ck) * a.H + h) * (a.vdim + 1) + a.vdim) * ds;
    const bool vec = a.dim % 4 == 0;
    const int wi = wave >> 1, wj = wave & 1, tok = tid >> 4, at = (tid & 15) * 4;
    const float scale = 1.f / sqrtf((float)a.dim);
    float4v acc[2][2] = {};
    float dot = 0.f;
    for (int d0 = 0; d0 < a.dim; d0 += 64) {
        float4 q[4], k[4];
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const float *row = a.cin + ((size_t)b * T + min(ck * CT + tok + 16 * i, T - 1)) * a.ldc;
            q[i] = take4(row + a.o_q + h * a.dim, d0 + at, a.dim, vec);
            k[i] = take4(row + a.o_k + h * a.dim, d0 + at, a.dim, vec);
        }
        const float nv = tid < 64 && d0 + tid < ds ? nc[d0 + tid] : 0.f;
        __syncthreads();
#pragma unroll
        for (int i = 0; i < 4; i++) {
            *reinterpret_cast<float4 *>(&Qs[(tok + 16 * i) * LDR + at]) = q[i];
            *reinterpret_cast<float4 *>(&Ks[(tok + 16 * i) * LDR + at]) = k[i];
        }
        if (tid < 64) ns[tid] = nv;
        __syncthreads();
        if (wj <= wi) tile_product<4>(Qs + 32 * wi * LDR, Ks + 32 * wj * LDR, c, r4, acc);
        // four threads per token, every fourth dimension each
#pragma unroll
        for (int e = 0; e < 16; e++) dot = fmaf(Qs[(tid >> 2) * LDR + (tid & 3) + 4 * e], ns[(tid & 3) + 4 * e], dot);
    }
    dot = dpp_add<0xB1>(dot);
    dot = dpp_add<0x4E>(dot);
    if ((tid & 3) == 0) qn[tid >> 2] = dot;
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int x = 0; x < 4; x++) {
            const int ti = 32 * wi + 16 * i + 4 * r4 + x;
            const float2 u = a.u[g0 + ti];
            float s = 0.f;
#pragma unroll
            for (int j = 0; j < 2; j++) {
                const int tj = 32 * wj + 16 * j + c;
                const float2 w = a.w[g0 + tj];
                const float e = tj <= ti && ti < nt ? expf((u.x + w.x) + (u.y + w.y)) * scale : 0.f;
                acc[i][j][x] *= e;
                s += acc[i][j][x];
            }
            s = group_sum<16>(s);
            if (c == 0) sums[wj][ti] = s;
        }
    __syncthreads();
    if (tid < CT) {
        const float f = a.cf[g0 + tid] * scale, n = fmaf(f, qn[tid], sums[0][tid] + sums[1][tid]);
        const float r = 1.f / (fmaxf(fabsf(n), a.em[g0 + tid]) + 1e-6f);
        rd[tid] = r;
        a.qf[g0 + tid] = f * r;
    }
    __syncthreads();
    float *P = a.P + (((size_t)b * chunks + ck) * a.H + h) * CT * CT;
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int x = 0; x < 4; x++) {
            const int ti = 32 * wi + 16 * i + 4 * r4 + x;
#pragma unroll
            for (int j = 0; j < 2; j++) P[ti * CT + 32 * wj + 16 * j + c] = acc[i][j][x] * rd[ti];
        }
}

// grid (tiles of 64 columns, chunks, H * B), block 256: outputs of a chunk's tokens in 64 columns, a wave 32 x 32 of them
__global__ __launch_bounds__(256) void k_mlstm_outputs(MlstmRows a, int chunks)
{
    __shared__ float As[CT * LDR], Bs[CT * LDR];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, r4 = lane >> 4;
    const int v0 = blockIdx.x * 64, ck = blockIdx.y, h = blockIdx.z % a.H, b = blockIdx.z / a.H, T = a.r.T, ds = up4(a.dim);
    const size_t g0 = (((size_t)b * a.H + h) * chunks + ck) * CT, part = ((size_t)b * chunks + ck) * a.H + h;
    const float *Sc = a.Sc + part * (a.vdim + 1) * ds, *P = a.P + part * CT * CT;
    const bool qvec = a.dim % 4 == 0, vvec = a.vdim % 4 == 0;
    const int wi = wave >> 1, wj = wave & 1, tok = tid >> 4, at = (tid & 15) * 4;
    float4v acc[2][2] = {};
    float4 x[4], y[4];
    auto fetch = [&](int d0) __attribute__((always_inline)) {      // d0 < dim: queries and state; behind: pairs and values
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int t = tok + 16 * i;
            const float *row = a.cin + ((size_t)b * T + min(ck * CT + t, T - 1)) * a.ldc;
            if (d0 < a.dim) {
                x[i] = take4(row + a.o_q + h * a.dim, d0 + at, a.dim, qvec);
                const float f = a.qf[g0 + t];
                x[i].x *= f; x[i].y *= f; x[i].z *= f; x[i].w *= f;
                y[i] = take4(Sc + (size_t)min(v0 + t, a.vdim) * ds, d0 + at, ds, true);
            } else {
                x[i] = *reinterpret_cast<const float4 *>(P + t * CT + at);
                y[i] = take4(row + a.o_v + h * a.vdim, v0 + at, a.vdim, vvec);
            }
        }
    };
    auto stage = [&]() __attribute__((always_inline)) {
        __syncthreads();
#pragma unroll
        for (int i = 0; i < 4; i++) {
            *reinterpret_cast<float4 *>(&As[(tok + 16 * i) * LDR + at]) = x[i];
            *reinterpret_cast<float4 *>(&Bs[(tok + 16 * i) * LDR + at]) = y[i];
        }
        __syncthreads();
    };
    fetch(0);
    for (int d0 = 0; d0 < a.dim; d0 += 64) {
        stage();
        fetch(d0 + 64);
        tile_product<4>(As + 32 * wi * LDR, Bs + 32 * wj * LDR, c, r4, acc);
    }
    stage();                                              // pairs by rows, values by steps
    const float *A = As + 32 * wi * LDR, *B = Bs + 32 * wj;
    for (int kb = 0; kb < 2 + 2 * wi; kb++) {             // later tokens weigh nothing
        float4v av[2];
#pragma unroll
        for (int i = 0; i < 2; i++) av[i] = *reinterpret_cast<const float4v *>(A + (16 * i + c) * LDR + 16 * kb + 4 * r4);
#pragma unroll
        for (int e = 0; e < 4; e++) {
            float bv[2];
#pragma unroll
            for (int j = 0; j < 2; j++) bv[j] = B[(16 * kb + 4 * r4 + e) * LDR + 16 * j + c];
#pragma unroll
            for (int i = 0; i < 2; i++)
#pragma unroll
                for (int j = 0; j < 2; j++) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(av[i][e], bv[j], acc[i][j], 0, 0, 0);
        }
    }
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int t = ck * CT + 32 * wi + 16 * i + 4 * r4 + e;
#pragma unroll
            for (int j = 0; j < 2; j++) {
                const int v = v0 + 32 * wj + 16 * j + c;
                if (t < T && v < a.vdim) a.o[((size_t)b * T + t) * a.H * a.vdim + h * a.vdim + v] = acc[i][j][e];
            }
        }
}

template <int G, int RPT>
void run_token(const MlstmRows &a)
{
    const int cols = 256 / G * RPT, nb = (a.vdim + cols - 1) / cols, dq = (a.dim + 4 * G - 1) / (4 * G) * 4 * G;
    LAUNCH((k_mlstm_token<G, RPT>), dim3(a.H * nb, a.r.B), dim3(256), (size_t)2 * dq * sizeof(float), a, nb, dq);
}

}  // namespace

void launch_mlstm(const MlstmRows &a)
{
    if (a.r.T == 1) {
        if (a.dim <= 32) run_token<8, 1>(a);
        else if (a.dim <= 64) run_token<16, 1>(a);
        else if (a.dim <= 128) run_token<32, 2>(a);
        else run_token<64, 4>(a);
        return;
    }
    const int chunks = mlstm_chunks(a.r.T);
    LAUNCH(k_mlstm_gates, dim3(a.H, a.r.B), dim3(256), 0, a, chunks);
    LAUNCH(k_mlstm_states, dim3((a.vdim + 64) / 64, (a.dim + 63) / 64, a.H * a.r.B), dim3(256), 0, a, chunks);
    LAUNCH(k_mlstm_pairs, dim3(chunks, a.H, a.r.B), dim3(256), 0, a, chunks);
    LAUNCH(k_mlstm_outputs, dim3((a.vdim + 63) / 64, chunks, a.H * a.r.B), dim3(256), 0, a, chunks);
}

}  // namespace lmhip
