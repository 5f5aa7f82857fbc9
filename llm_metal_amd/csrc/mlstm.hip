// mLSTM: a matrix memory per head with exponential gates.  With the logarithms i, f of the input and forget gate and the
// running maximum m_t = max(f_t + m_(t-1), i_t),
//     S_t = e^(f_t + m_(t-1) - m_t) S_(t-1) + e^(i_t - m_t) k_t v_t^T         n_t likewise with k_t alone
//     o_t = S_t^T q_t / (max(|n_t . q_t|, e^(-m_t)) + 1e-6)
// Everything here is fp32, the matrix instructions included.
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

// grid (H, B), block 64 NW: a wave takes a chunk of 64 tokens, a lane one of them.  Per token: u = F - m and w = i - F as sums
// of two floats, cf = e^(F + m_c - m), wk = e^(F_L - F + i - m_L), em = e^(-m); per chunk gk = e^(F_L + m_c - m_L).
template <int NW>
__global__ __launch_bounds__(64 * NW) void k_mlstm_gates(MlstmRows a, int chunks)
{
    __shared__ float wa[NW], wb[NW];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.x, b = blockIdx.y, T = a.r.T;
    const size_t base = ((size_t)b * a.H + h) * chunks * CT;
    float carry = a.r.pos > 0 ? *m_slot(a, a.r.pos, b, h) : 0.f;
    for (int t0 = 0; t0 < T; t0 += 64 * NW) {
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
        for (int w = 0; w < NW; w++) carry = fmaxf(wa[w] + carry, wb[w]);
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

// Workgroup ids go to the eight XCDs in turn.  Place of this workgroup in a list of n of which each XCD takes a contiguous
// share, so that what neighbours of the list read lies in one L2.
__device__ __forceinline__ int xcd_share(int id, int n)
{
    const int x = id & 7, rest = n & 7;
    return x * (n >> 3) + min(x, rest) + (id >> 3);
}

// Four consecutive entries from column d on of a row of n: asked for at places that exist (nothing waits here), and those
// behind the row's end zeroed when they are used.  VEC: rows start on 16 bytes and n % 4 == 0.
template <bool VEC>
__device__ __forceinline__ float4 ask4(const float *row, int d, int n)
{
    if (VEC) return *reinterpret_cast<const float4 *>(row + min(d, n - 4));
    float4 v;
#pragma unroll
    for (int e = 0; e < 4; e++) (&v.x)[e] = row[min(d + e, n - 1)];
    return v;
}
__device__ __forceinline__ float4 kept4(float4 v, int d, int n, float f)
{
    return make_float4(d < n ? v.x * f : 0.f, d + 1 < n ? v.y * f : 0.f, d + 2 < n ? v.z * f : 0.f, d + 3 < n ? v.w * f : 0.f);
}

// Operands in LDS for v_mfma_f32_16x16x4_f32 (A: lane -> row lane & 15; B: lane -> column lane & 15; both: reduction index
// lane >> 4; accumulator: column lane & 15, rows 4 (lane >> 4) + 0 .. 3).  The reduction may go in any order common to both.
//   by rows [row][LDR]: four reduction steps of a lane are one 16-byte read, indices 16 kb + 4 (lane >> 4) + 0 .. 3
//   by steps [index][LDS_]: sixteen rows lie side by side
constexpr int LDR = CT + 4, LDK = CT + 16;

// The state ahead of a chunk lies in tiles of 16 columns x 16 dimensions, [column tile][dimension tile][lane][4]: lane ->
// column lane & 15, dimensions 4 (lane >> 4) + 0 .. 3 -- as the accumulators that make it and the operand that takes it hold
// it; what lies beyond the head is zero.  Behind the tiles the normaliser, in four parts of [dimension tiles][16].
__device__ __forceinline__ int v_tiles(const MlstmRows &a) { return (a.vdim + 15) / 16; }
__device__ __forceinline__ int d_tiles(const MlstmRows &a) { return (a.dim + 15) / 16; }
__device__ __forceinline__ float *state_ahead(const MlstmRows &a, int chunks, int b, int ck, int h)
{
    return a.Sc + (((size_t)b * chunks + ck) * a.H + h) * (v_tiles(a) * 256 + 64) * d_tiles(a);
}

// grid (nv tiles of 64 columns * nd tiles of 64 dimensions * H * B), block 256: a workgroup takes one 64 x 64 tile of a head's
// state through the chunks in order, a wave a quarter of it.  Those of the first columns also take their dimensions of the
// normaliser along, each wave over a quarter of the tokens: their sum is left to whoever reads it.
template <bool VEC>
__global__ __launch_bounds__(256) void k_mlstm_states(MlstmRows a, int chunks, int nv, int nd)
{
    __shared__ float Ks[CT * LDK], Vs[CT * LDK];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, r4 = lane >> 4;
    const int id = xcd_share(blockIdx.x, gridDim.x), hb = id / (nv * nd), h = hb % a.H, b = hb / a.H, T = a.r.T, ds = up4(a.dim);
    const int v0 = id % nv * 64, d0 = id / nv % nd * 64, wv = v0 + (wave & 1) * 32, wd = d0 + (wave >> 1) * 32;
    const int VT = v_tiles(a), DT = d_tiles(a);
    const bool norm = v0 == 0;
    float n = norm && wave == 0 && a.r.pos > 0 && d0 + lane < a.dim ? n_slot(a, a.r.pos, b, h)[d0 + lane] : 0.f;
    // dimensions d .. d + 3 of column v of the lasting state
    auto place = [&](int v, int d) __attribute__((always_inline)) {
        return reinterpret_cast<float4v *>(a.S + (((size_t)b * a.H + h) * a.vdim + v) * ds + d);
    };
    float4v S[2][2];                                      // [dimensions][columns]
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int j = 0; j < 2; j++) {
            const int v = wv + 16 * j + c, d = wd + 16 * i + 4 * r4;
            S[i][j] = float4v{0.f, 0.f, 0.f, 0.f};
            if (a.r.pos > 0 && d < ds && v < a.vdim) S[i][j] = *place(v, d);
        }
    const int tok = tid >> 4, at = (tid & 15) * 4;        // four tokens of a thread, sixteen apart
    struct Set { float4 k[4], v[4]; float w[4], g; };
    auto fetch = [&](Set &x, int ck_) __attribute__((always_inline)) {
        const int ck = min(ck_, chunks - 1);
        const size_t part = ((size_t)b * a.H + h) * chunks + ck;
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const float *row = a.cin + ((size_t)b * T + min(ck * CT + tok + 16 * i, T - 1)) * a.ldc;
            x.k[i] = ask4<VEC>(row + a.o_k + h * a.dim, d0 + at, a.dim);
            x.v[i] = ask4<VEC>(row + a.o_v + h * a.vdim, v0 + at, a.vdim);
            x.w[i] = a.wk[part * CT + tok + 16 * i];      // 0 past the end
        }
        x.g = a.gk[part];
    };
    auto take = [&](const Set &x, int ck) __attribute__((always_inline)) {
        __syncthreads();
#pragma unroll
        for (int i = 0; i < 4; i++) {
            *reinterpret_cast<float4 *>(&Ks[(tok + 16 * i) * LDK + at]) = kept4(x.k[i], d0 + at, a.dim, x.w[i]);
            *reinterpret_cast<float4 *>(&Vs[(tok + 16 * i) * LDK + at]) = kept4(x.v[i], v0 + at, a.vdim, 1.f);
        }
        const float g = x.g;
        __syncthreads();
        float *out = state_ahead(a, chunks, b, ck, h) + lane * 4;
#pragma unroll
        for (int i = 0; i < 2; i++)
#pragma unroll
            for (int j = 0; j < 2; j++) {
                const int vt = (wv >> 4) + j, dt = (wd >> 4) + i;
                if (vt < VT && dt < DT) *reinterpret_cast<float4v *>(out + (size_t)(vt * DT + dt) * 256) = S[i][j];
                S[i][j] *= g;
            }
        if (norm) {
            if (d0 + lane < 16 * DT) (out - lane * 4)[(size_t)VT * DT * 256 + wave * DT * 16 + d0 + lane] = n;
            n *= g;
#pragma unroll
            for (int t = 0; t < CT / 4; t++) n += Ks[(wave * (CT / 4) + t) * LDK + lane];
        }
        const float *kp = Ks + r4 * LDK + (wave >> 1) * 32 + c, *vp = Vs + r4 * LDK + (wave & 1) * 32 + c;
#pragma unroll
        for (int s = 0; s < CT / 4; s++) {
            float av[2], bv[2];
#pragma unroll
            for (int i = 0; i < 2; i++) { av[i] = kp[4 * s * LDK + 16 * i]; bv[i] = vp[4 * s * LDK + 16 * i]; }
#pragma unroll
            for (int i = 0; i < 2; i++)
#pragma unroll
                for (int j = 0; j < 2; j++) S[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(av[i], bv[j], S[i][j], 0, 0, 0);
        }
    };
    constexpr int SETS = 3;                               // a chunk is asked for two chunks ahead
    Set x[SETS];
#pragma unroll
    for (int n = 0; n < SETS - 1; n++) fetch(x[n], n);
    for (int ck = 0; ck < chunks; ck += SETS)
#pragma unroll
        for (int n = 0; n < SETS; n++) {
            if (ck + n >= chunks) break;                  // uniform
            fetch(x[(n + SETS - 1) % SETS], ck + n + SETS - 1);
            take(x[n], ck + n);
        }
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int j = 0; j < 2; j++) {
            const int v = wv + 16 * j + c, d = wd + 16 * i + 4 * r4;
            if (d < ds && v < a.vdim) *place(v, d) = S[i][j];
        }
    if (!norm) return;
    __syncthreads();
    Ks[tid] = n;
    __syncthreads();
    if (tid < 64 && d0 + tid < ds) n_slot(a, a.r.pos + T, b, h)[d0 + tid] = (Ks[tid] + Ks[64 + tid]) + (Ks[128 + tid] + Ks[192 + tid]);
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
template <bool VEC>
__global__ __launch_bounds__(256) void k_mlstm_pairs(MlstmRows a, int chunks)
{
    __shared__ float Qs[CT * LDR], Ks[CT * LDR], ns[CT], sums[2][CT], qn[CT], rd[CT];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, r4 = lane >> 4;
    const int ck = blockIdx.x, h = blockIdx.y, b = blockIdx.z, T = a.r.T, nt = min(CT, T - ck * CT);
    const size_t g0 = (((size_t)b * a.H + h) * chunks + ck) * CT;
    const int DT16 = d_tiles(a) * 16;
    const float *nc = state_ahead(a, chunks, b, ck, h) + (size_t)v_tiles(a) * DT16 * 16;
    const int wi = wave >> 1, wj = wave & 1, tok = tid >> 4, at = (tid & 15) * 4;
    const float scale = 1.f / sqrtf((float)a.dim);
    float4v acc[2][2] = {};
    float dot = 0.f;
    float4 q[4], k[4];
    float nv = 0.f;
    auto fetch = [&](int d0) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const float *row = a.cin + ((size_t)b * T + min(ck * CT + tok + 16 * i, T - 1)) * a.ldc;
            q[i] = ask4<VEC>(row + a.o_q + h * a.dim, d0 + at, a.dim);
            k[i] = ask4<VEC>(row + a.o_k + h * a.dim, d0 + at, a.dim);
        }
        const int d = min(d0 + (tid & 63), a.dim - 1);
        nv = (nc[d] + nc[DT16 + d]) + (nc[2 * DT16 + d] + nc[3 * DT16 + d]);
    };
    fetch(0);
    for (int d0 = 0; d0 < a.dim; d0 += 64) {
        __syncthreads();
#pragma unroll
        for (int i = 0; i < 4; i++) {
            *reinterpret_cast<float4 *>(&Qs[(tok + 16 * i) * LDR + at]) = kept4(q[i], d0 + at, a.dim, 1.f);
            *reinterpret_cast<float4 *>(&Ks[(tok + 16 * i) * LDR + at]) = kept4(k[i], d0 + at, a.dim, 1.f);
        }
        if (tid < 64) ns[tid] = d0 + tid < a.dim ? nv : 0.f;
        __syncthreads();
        if (d0 + 64 < a.dim) fetch(d0 + 64);
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

// grid (nv tiles of 64 columns * chunks * H * B), block 256: outputs of a chunk's tokens in 64 columns, a wave 32 x 32 of them
template <bool VEC>
__global__ __launch_bounds__(256) void k_mlstm_outputs(MlstmRows a, int chunks, int nv)
{
    __shared__ float As[CT * LDR], Bs[CT * LDR];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, r4 = lane >> 4;
    const int id = xcd_share(blockIdx.x, gridDim.x), hb = id / (nv * chunks), h = hb % a.H, b = hb / a.H, T = a.r.T;
    const int v0 = id % nv * 64, ck = id / nv % chunks;
    const size_t g0 = (((size_t)b * a.H + h) * chunks + ck) * CT;
    const int wi = wave >> 1, wj = wave & 1, tok = tid >> 4, at = (tid & 15) * 4, VT = v_tiles(a), DT = d_tiles(a);
    const float *P = a.P + (((size_t)b * chunks + ck) * a.H + h) * CT * CT;
    const float *Sc[2];
#pragma unroll
    for (int j = 0; j < 2; j++) Sc[j] = state_ahead(a, chunks, b, ck, h) + (size_t)min((v0 >> 4) + 2 * wj + j, VT - 1) * DT * 256 + lane * 4;
    float4v acc[2][2] = {}, B0[4][2], B1[4][2];
    float4 x[4], y[4], p[4];
    float f[4];
#pragma unroll
    for (int i = 0; i < 4; i++) f[i] = a.qf[g0 + tok + 16 * i];
    auto row = [&](int i) __attribute__((always_inline)) { return a.cin + ((size_t)b * T + min(ck * CT + tok + 16 * i, T - 1)) * a.ldc; };
    auto ask = [&](int d0, float4v (&B)[4][2]) __attribute__((always_inline)) {        // queries, and the state as an operand
#pragma unroll
        for (int i = 0; i < 4; i++) x[i] = ask4<VEC>(row(i) + a.o_q + h * a.dim, d0 + at, a.dim);
#pragma unroll
        for (int kb = 0; kb < 4; kb++)
#pragma unroll
            for (int j = 0; j < 2; j++) B[kb][j] = *reinterpret_cast<const float4v *>(Sc[j] + (size_t)min((d0 >> 4) + kb, DT - 1) * 256);
    };
    auto use = [&](int d0, const float4v (&B)[4][2], float4v (&next)[4][2]) __attribute__((always_inline)) {
        __syncthreads();
#pragma unroll
        for (int i = 0; i < 4; i++) *reinterpret_cast<float4 *>(&As[(tok + 16 * i) * LDR + at]) = kept4(x[i], d0 + at, a.dim, f[i]);
        __syncthreads();
        if (d0 + 64 < a.dim) ask(d0 + 64, next);
#pragma unroll
        for (int kb = 0; kb < 4; kb++) {                  // (dimensions beyond the head's: the queries are zero)
            float4v av[2];
#pragma unroll
            for (int i = 0; i < 2; i++) av[i] = *reinterpret_cast<const float4v *>(As + (32 * wi + 16 * i + c) * LDR + 16 * kb + 4 * r4);
#pragma unroll
            for (int e = 0; e < 4; e++)
#pragma unroll
                for (int i = 0; i < 2; i++)
#pragma unroll
                    for (int j = 0; j < 2; j++) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(av[i][e], B[kb][j][e], acc[i][j], 0, 0, 0);
        }
    };
    ask(0, B0);
#pragma unroll
    for (int i = 0; i < 4; i++) {                         // pairs and values, for the end
        p[i] = *reinterpret_cast<const float4 *>(P + (tok + 16 * i) * CT + at);
        y[i] = ask4<VEC>(row(i) + a.o_v + h * a.vdim, v0 + at, a.vdim);
    }
    for (int d0 = 0; d0 < a.dim; d0 += 128) {
        use(d0, B0, B1);
        if (d0 + 64 < a.dim) use(d0 + 64, B1, B0);
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 4; i++) {                         // pairs by rows, values by steps
        *reinterpret_cast<float4 *>(&As[(tok + 16 * i) * LDR + at]) = p[i];
        *reinterpret_cast<float4 *>(&Bs[(tok + 16 * i) * LDR + at]) = kept4(y[i], v0 + at, a.vdim, 1.f);
    }
    __syncthreads();
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
    if (chunks <= 4) LAUNCH(k_mlstm_gates<4>, dim3(a.H, a.r.B), dim3(256), 0, a, chunks);
    else LAUNCH(k_mlstm_gates<16>, dim3(a.H, a.r.B), dim3(1024), 0, a, chunks);
    const int nv = (a.vdim + 63) / 64, nd = (a.dim + 63) / 64;
    const dim3 states(nv * nd * a.H * a.r.B), pairs(chunks, a.H, a.r.B), outputs(nv * chunks * a.H * a.r.B);
#define CHUNKS(VEC_) do { LAUNCH((k_mlstm_states<VEC_>), states, dim3(256), 0, a, chunks, nv, nd); LAUNCH((k_mlstm_pairs<VEC_>), pairs, dim3(256), 0, a, chunks); \
                          LAUNCH((k_mlstm_outputs<VEC_>), outputs, dim3(256), 0, a, chunks, nv); } while (0)
    if (a.dim % 4 == 0 && a.vdim % 4 == 0) CHUNKS(true); else CHUNKS(false);
#undef CHUNKS
}

}  // namespace lmhip
